"""Plain CPU statement of the hybrid decoder family (``trimkv_amd/fusitar.py``): windowed attention with kept first
tokens, mLSTM matrix memory, grouped sigmoid routing over squared-ReLU experts, norms behind the sublayers.

One function per mechanism, one sequence at a time, no cache and no batching; everything is computed in ``dtype``
(float64 unless a caller asks otherwise).  It shares no code with the product path: weights arrive as a plain
``name -> tensor`` dictionary and the configuration as the dictionary that config.json holds.

Notation: t, s count tokens of one sequence from 0; x is the residual stream [T, width].
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x divided by the root of (mean square over the last axis + eps)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def window_visible(i: int, j: int, size: int, keep_first: int) -> bool:
    return j <= i and (i - j < size or j < keep_first)


def window_attention(q, k, v, scale: float, size: int, keep_first: int) -> torch.Tensor:
    """q [T,H,D], k [T,G,D], v [T,G,Dv] -> [T,H,Dv]; query head h reads key/value head h // (H // G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = q.new_zeros(T, H, v.shape[2])
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    seen = (j <= i) & ((i - j < size) | (j < keep_first))
    for h in range(H):
        g = h // per
        score = (q[:, h] @ k[:, g].T) * scale
        score = score.masked_fill(~seen, -math.inf)
        out[:, h] = torch.softmax(score, dim=-1) @ v[:, g]
    return out


def attention_mixer(h, w: Dict[str, torch.Tensor], cfg: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = (rms(h @ w["q"].T, eps) * w["q.norm"]).view(T, H, D)          # over all heads at once
    k = (rms(h @ w["k"].T, eps) * w["k.norm"]).view(T, G, D)
    v = (h @ w["v"].T).view(T, G, Dv)
    o = window_attention(q, k, v, cfg["scale"], cfg["mask"]["size"], cfg["mask"]["keep_first"]).reshape(T, H * Dv)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def soft_cap(z, cap: float):
    return cap * torch.tanh(z / cap)


def mlstm_scan(q, k, v, log_i, log_f, state: Optional[tuple] = None):
    """Token by token: q, k [T,H,D] (q already scaled), v [T,H,Dv], log_i, log_f [T,H].  Returns outputs [T,H,Dv] and the
    state (S [H,D,Dv], n [H,D], m [H]) behind the last token.  ``state`` None: the zero state with m = 0."""
    T, H, D = q.shape
    if state is None:
        state = (q.new_zeros(H, D, v.shape[2]), q.new_zeros(H, D), q.new_zeros(H))
    S, n, m = state
    out = q.new_zeros(T, H, v.shape[2])
    for t in range(T):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = m_new
        num = torch.einsum("hdv,hd->hv", S, q[t])
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = num / den[:, None]
    return out, (S, n, m)


def mlstm_mixer(h, w, cfg: dict, eps: float, state=None, want_state: bool = False):
    T = h.shape[0]
    H, D, Dv, cap = cfg["heads"], cfg["dim"], cfg["vdim"], cfg["gate_cap"]
    q = (h @ w["q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w["k"].T).view(T, H, D)
    v = (h @ w["v"].T).view(T, H, Dv)
    log_i = soft_cap(h @ w["i"].T + w["i.b"], cap)
    log_f = torch.nn.functional.logsigmoid(soft_cap(h @ w["f"].T + w["f.b"], cap))
    o, state = mlstm_scan(q, k, v, log_i, log_f, state)
    y = (rms(o, eps).reshape(T, H * Dv) * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T
    return (y, state) if want_state else y


def choose_experts(z, correction, top: int, count: int, keep: int):
    """Router logits z [T,E] -> (expert ids [T,top], weights [T,top])."""
    s = torch.sigmoid(z)
    ids, weights = [], []
    E = z.shape[1]
    per = E // count
    for t in range(z.shape[0]):
        choice = (s[t] + correction).tolist()
        group = [sum(sorted(choice[g * per:(g + 1) * per], reverse=True)[:2]) for g in range(count)]
        best = sorted(range(count), key=lambda g: -group[g])[:keep]
        open_ = [e for e in range(E) if e // per in best]
        chosen = sorted(open_, key=lambda e: -choice[e])[:top]
        ids.append(chosen)
        weights.append(s[t, chosen])
    return torch.tensor(ids), torch.stack(weights)


def expert(h, up, down):
    a = torch.relu(h @ up.T)
    return (a * a) @ down.T


def moe(h, w, cfg: dict):
    r = cfg["router"]
    ids, weights = choose_experts(h @ w["router"].T, w["correction"], r["top"], r["groups"]["count"], r["groups"]["keep"])
    out = torch.zeros_like(h)
    for e in range(r["experts"]):
        t, c = (ids == e).nonzero(as_tuple=True)
        if len(t):
            out[t] += weights[t, c][:, None] * expert(h[t], w[f"e{e}.up"], w[f"e{e}.down"])
    return out


def _under(state: Dict[str, torch.Tensor], prefix: str, dtype) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v.to(dtype) for k, v in state.items() if k.startswith(prefix)}


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64, layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  ``layers_out`` receives the residual stream behind every layer."""
    eps = config["norm"]["eps"]
    table = weights["embed"].to(dtype)
    x = table[torch.tensor(tokens)] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        mix = _under(weights, f"l{i}.mix.", dtype)
        y = {"attention": attention_mixer, "mlstm": mlstm_mixer}[layer["type"]](x, mix, layer["mixer"], eps)
        x = x + rms(y, eps) * weights[f"l{i}.norm1"].to(dtype)
        if layer.get("mlp") is not None:
            y = moe(x, _under(weights, f"l{i}.mlp.", dtype), layer["mlp"])
            x = x + rms(y, eps) * weights[f"l{i}.norm2"].to(dtype)
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * weights["final.norm"].to(dtype)) @ table.T
