"""The Fusitar design: windowed attention and mLSTM layers in any order, routed squared-ReLU experts, norms on the
sublayers' outputs, scaled embedding and tied head.  Configuration and names only; the layers are in ``hybrid.py``."""
from __future__ import annotations

from dataclasses import dataclass
from typing import List

from .hybrid import FEED_FORWARDS, MIXERS, HybridForCausalLM

_MIXER_KEYS = {"attention": ("heads", "kv_heads", "dim", "vdim", "scale", "mask"), "mlstm": ("heads", "dim", "vdim", "gate_cap")}


@dataclass
class FusitarConfig:
    """Fields of config.json: ``vocab``, ``width``, ``embedding.scale``, ``norm.eps`` and ``layers`` (each with ``type``,
    ``mixer`` and ``mlp``), under this package's names."""
    vocab_size: int
    hidden_size: int
    embedding_scale: float
    norm_eps: float
    layers: List[dict]
    architecture: str = "Fusitar"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: dict, **overrides) -> "FusitarConfig":
        fields = dict(vocab_size=d["vocab"], hidden_size=d["width"], embedding_scale=float(d["embedding"]["scale"]),
                      norm_eps=float(d["norm"]["eps"]), layers=list(d["layers"]))
        fields.update({k: v for k, v in overrides.items() if k in fields})
        cfg = cls(**fields)
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a Fusitar model needs at least one layer")
        for i, layer in enumerate(self.layers):
            kind, m, mlp = layer.get("type"), layer.get("mixer", {}), layer.get("mlp")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r} (one of {sorted(MIXERS)})")
            lacking = [k for k in _MIXER_KEYS[kind] if k not in m]
            if lacking:
                raise ValueError(f"layer {i}: the {kind} mixer lacks {lacking}")
            if kind == "attention":
                if m["heads"] % m["kv_heads"]:
                    raise ValueError(f"layer {i}: {m['heads']} query heads do not divide among {m['kv_heads']} key/value heads")
                if m["mask"]["size"] < 1 or m["mask"]["keep_first"] < 0:
                    raise ValueError(f"layer {i}: bad window {m['mask']}")
            if mlp is None:
                continue
            if mlp.get("kind") not in FEED_FORWARDS:
                raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r} (one of {sorted(FEED_FORWARDS)})")
            r = mlp["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            if r["experts"] % g["count"] or not 1 <= g["keep"] <= g["count"] or not 1 <= r["top"] <= g["keep"] * (r["experts"] // g["count"]):
                raise ValueError(f"layer {i}: router {r} cannot choose {r['top']} experts")


class FusitarForCausalLM(HybridForCausalLM):
    config_cls = FusitarConfig
