"""Plain CPU statement of the Siterax design (``trimkv_amd/siterax.py``): sliding-window attention with rotary positions,
normed heads, a unit term in the softmax denominator and one output gate per head; gated dense feed-forward; norms on both
sides of every sublayer; a run of layers that is passed several times; soft-capped logits.

One function per mechanism, one sequence at a time, no cache and no batching, everything in ``dtype`` (float64 unless a
caller asks otherwise).  It shares no code with the product path: weights arrive as a plain ``name -> tensor`` dictionary
and the configuration as the dictionary that config.json holds.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from .hybrid_ref import rms, soft_cap


def rotation_frequencies(dims: int, base: float, factor: float) -> torch.Tensor:
    """Radians per position of the dims / 2 rotated pairs; ``factor`` stretches every wavelength."""
    return torch.tensor([base ** (-2.0 * i / dims) / factor for i in range(dims // 2)], dtype=torch.float64)


def rotate(x: torch.Tensor, first: int, dims: int, base: float, factor: float) -> torch.Tensor:
    """x [T, heads, D], its first token at position ``first``: pair (i, i + dims / 2) turns by position * frequency i."""
    half = dims // 2
    out = x.clone()
    freq = rotation_frequencies(dims, base, factor)
    for t in range(x.shape[0]):
        a = (first + t) * freq
        c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
        u, v = x[t, :, :half], x[t, :, half:dims]
        out[t, :, :half] = u * c - v * s
        out[t, :, half:dims] = v * c + u * s
    return out


def sink_weights(score: torch.Tensor) -> torch.Tensor:
    """exp(score) / (1 + sum exp(score)) over the last axis; -inf: not seen."""
    top = score.amax(-1, keepdim=True).clamp(min=0.0)
    e = torch.exp(score - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def sink_window_attention(q, k, v, scale: float, size: int) -> torch.Tensor:
    """q [T,H,D], k [T,G,D], v [T,G,Dv] -> [T,H,Dv]; token i sees the ``size`` newest tokens up to itself."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    age = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    hidden = (age < 0) | (age >= size)
    out = q.new_zeros(T, H, v.shape[2])
    for h in range(H):
        score = ((q[:, h] @ k[:, h // per].T) * scale).masked_fill(hidden, -float("inf"))
        out[:, h] = sink_weights(score) @ v[:, h // per]
    return out


def project(h, w: Dict[str, torch.Tensor], name: str, heads: int) -> torch.Tensor:
    return (h @ w[name].T + w[name + ".b"]).view(h.shape[0], heads, -1)


def head_gate(o, h, w) -> torch.Tensor:
    """o [T,H,Dv] times one sigmoid per head."""
    return o * torch.sigmoid(h @ w["g"].T)[:, :, None]


def attention(h, w: Dict[str, torch.Tensor], cfg: dict, eps: float) -> torch.Tensor:
    rot = cfg["rot"]
    turn = lambda x: rotate(x, 0, rot["dims"], rot["base"], rot["scaling"]["factor"])
    q = turn(rms(project(h, w, "q", cfg["heads"]), eps) * w["q.norm"])
    k = turn(rms(project(h, w, "k", cfg["kv_heads"]), eps) * w["k.norm"])
    o = sink_window_attention(q, k, project(h, w, "v", cfg["kv_heads"]), cfg["scale"], cfg["mask"]["size"])
    return head_gate(o, h, w).reshape(h.shape[0], -1) @ w["o"].T


def gated_mlp(h, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    z = h @ w["gate"].T
    return (z / (1.0 + torch.exp(-z)) * (h @ w["up"].T)) @ w["down"].T


def layer_order(count: int, loop: Optional[dict]) -> List[tuple]:
    """(layer, whether a further pass starts with it), in the order of execution."""
    if not loop:
        return [(i, False) for i in range(count)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for n in range(loop["times"]):
        out += [(i, n > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, count)]


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64, layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  ``layers_out`` receives the residual stream behind every layer that runs."""
    eps, m = config["norm"]["eps"], config["residual_mult"]
    W = {k: v.to(dtype) for k, v in weights.items()}
    under = lambda p: {k[len(p):]: v for k, v in W.items() if k.startswith(p)}
    start = W["embed"][torch.tensor(tokens)]
    x = start
    for i, again in layer_order(len(config["layers"]), config.get("loop")):
        layer = config["layers"][i]
        if again:
            x = x + start
        norm = lambda name, y: rms(y, eps) * W[f"l{i}.{name}"]
        x = x + m * norm("norm1b", attention(norm("norm1", x), under(f"l{i}.mix."), layer["mixer"], eps))
        if layer.get("mlp") is not None:
            x = x + m * norm("norm2b", gated_mlp(norm("norm2", x), under(f"l{i}.mlp.")))
        if layers_out is not None:
            layers_out.append(x.clone())
    return soft_cap((rms(x, eps) * W["final.norm"]) @ W["head"].T, config["logit_softcap"])
