"""The Fusitar design: windowed attention and mLSTM layers in any order, routed squared-ReLU experts, norms on the
sublayers' outputs, scaled embedding and tied head.  Configuration and names only; the layers are in ``hybrid.py``."""
from __future__ import annotations

from dataclasses import dataclass

from .hybrid import HybridConfig, HybridForCausalLM


@dataclass
class FusitarConfig(HybridConfig):
    """Fields of config.json: ``vocab``, ``width``, ``embedding.scale``, ``norm.eps`` and ``layers`` (each with ``type``,
    ``mixer`` and ``mlp``), under this package's names."""
    architecture: str = "Fusitar"

    @classmethod
    def from_dict(cls, d: dict, **overrides) -> "FusitarConfig":
        fields = dict(vocab_size=d["vocab"], hidden_size=d["width"], embedding_scale=float(d["embedding"]["scale"]),
                      norm_eps=float(d["norm"]["eps"]), layers=list(d["layers"]))
        fields.update({k: v for k, v in overrides.items() if k in fields})
        cfg = cls(**fields)
        cfg.validate()
        return cfg


class FusitarForCausalLM(HybridForCausalLM):
    config_cls = FusitarConfig
