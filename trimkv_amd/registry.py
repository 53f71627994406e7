"""Which model class a checkpoint directory asks for, and what every loader shares: reading config.json and the tensors."""
from __future__ import annotations

import glob
import importlib
import json
import os
from typing import Dict

import torch

# architecture name in config.json (``architecture``, or an entry of HF's ``architectures``) -> (module, class)
MODELS = {
    "Fusitar": ("fusitar", "FusitarForCausalLM"),
    "Siterax": ("siterax", "SiteraxForCausalLM"),
    "TrimKVQwen3ForCausalLM": ("qwen3", "TrimKVQwen3ForCausalLM"),
    "Qwen3ForCausalLM": ("qwen3", "TrimKVQwen3ForCausalLM"),
    "TrimKVLlamaForCausalLM": ("llama", "TrimKVLlamaForCausalLM"),
    "LlamaForCausalLM": ("llama", "TrimKVLlamaForCausalLM"),
    "TrimKVPhi3ForCausalLM": ("phi3", "TrimKVPhi3ForCausalLM"),
    "Phi3ForCausalLM": ("phi3", "TrimKVPhi3ForCausalLM"),
}


def read_config(directory: str) -> dict:
    if not os.path.isdir(directory):
        raise ValueError(f"Path {directory} does not exist.")
    with open(os.path.join(directory, "config.json")) as f:
        return json.load(f)


def model_class(config: dict):
    """The class for a config.json dictionary."""
    names = [config["architecture"]] if "architecture" in config else list(config.get("architectures") or [])
    for name in names:
        if name in MODELS:
            module, cls = MODELS[name]
            return getattr(importlib.import_module(f"{__package__}.{module}"), cls)
    raise ValueError(f"no model for architecture {names or None} (known: {', '.join(sorted(MODELS))})")


def from_pretrained(directory: str, **kwargs):
    """Load whatever model the directory holds (keyword arguments as in the class's own ``from_pretrained``)."""
    return model_class(read_config(directory)).from_pretrained(directory, **kwargs)


def load_checkpoint_tensors(directory: str) -> Dict[str, torch.Tensor]:
    """All tensors of a local checkpoint directory: ``*.safetensors`` shards, else ``pytorch_model*.bin`` read with
    ``weights_only=True`` (nothing in the files is executed)."""
    shards = sorted(glob.glob(os.path.join(directory, "*.safetensors")))
    state = {}
    if shards:
        from safetensors.torch import load_file
        for f in shards:
            state.update(load_file(f))
        return state
    for f in sorted(glob.glob(os.path.join(directory, "pytorch_model*.bin"))):
        state.update(torch.load(f, map_location="cpu", weights_only=True))
    if not state:
        raise FileNotFoundError(f"no *.safetensors or pytorch_model*.bin under {directory}")
    return state
