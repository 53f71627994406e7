"""The Siterax design: sliding-window attention with rotary positions, biases, heads normed one by one, a softmax sink and a gate
per head; gated dense feed-forwards; norms on both sides of every sublayer; a run of layers that is passed several times with
the embedding added in between; untied head with soft-capped logits.  Configuration and names only; the layers are in
``hybrid.py``."""
from __future__ import annotations

from dataclasses import dataclass

from .hybrid import HybridConfig, HybridForCausalLM

# what the design fixes about its attention, beside the sizes that config.json gives
ATTENTION_FORM = {"qk_norm": "head", "bias": True, "gate": "head", "sink": True}


@dataclass
class SiteraxConfig(HybridConfig):
    """Fields of config.json: ``vocab``, ``width``, ``norm.eps``, ``residual_mult``, ``loop``, ``logit_softcap`` and ``layers`` (each
    with ``type``, ``mixer`` and ``mlp``), under this package's names."""
    architecture: str = "Siterax"

    @classmethod
    def from_dict(cls, d: dict, **overrides) -> "SiteraxConfig":
        layers = []
        for i, layer in enumerate(d["layers"]):
            mixer, mlp = layer.get("mixer") or {}, layer.get("mlp")
            if layer.get("type") != "attention":
                raise ValueError(f"layer {i}: unknown mixer {layer.get('type')!r} (Siterax has attention only)")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r} (Siterax has dense ones only)")
            if "rot" not in mixer:
                raise ValueError(f"layer {i}: the attention mixer lacks ['rot']")
            layers.append(dict(layer, mixer={**mixer, **ATTENTION_FORM}))
        fields = dict(vocab_size=d["vocab"], hidden_size=d["width"], norm_eps=float(d["norm"]["eps"]), layers=layers, tied_head=False, norms="both",
                      residual_mult=float(d["residual_mult"]), loop=d.get("loop"), logit_softcap=float(d["logit_softcap"]))
        fields.update({k: v for k, v in overrides.items() if k in fields})
        cfg = cls(**fields)
        cfg.validate()
        return cfg


class SiteraxForCausalLM(HybridForCausalLM):
    config_cls = SiteraxConfig
