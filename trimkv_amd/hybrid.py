"""Decoders whose layers mix windowed attention with recurrent layers and routed experts, on the kernels of
libtrimkv_hybrid.so.

A layer is a mixer and, optionally, a feed-forward; both are looked up by kind (``MIXERS``, ``FEED_FORWARDS``) and bring
their sizes as parameters, so another design of the same kind is another configuration.  The residual stream is fp32; the
norms sit behind the sublayers, which read the stream itself (``x += norm(sublayer(x))``).  Matrices and activations are bf16
or fp32 throughout; norm weights, biases and corrections are fp32.

Batches are packed: the tokens of unequal sequences lie one after the other, no padding is computed.  The same forward serves
prompts, portions of prompts and decode steps; what a sequence leaves behind is in a ``HybridCache``.
"""
from __future__ import annotations

from types import SimpleNamespace
from typing import Dict, List, Optional, Sequence

import torch
from torch import nn
import torch.nn.functional as F

from . import _lib, hybrid_ops as ops
from .generation import GreedyGeneration
from .hybrid_cache import HybridCache


def _param(*shape, dtype) -> nn.Parameter:
    return nn.Parameter(torch.zeros(*shape, dtype=dtype), requires_grad=False)


class PackedLinear(nn.Module):
    """Several matrices over the same input as one weight; ``section(name)`` is the rows of one of them."""

    def __init__(self, sections: Dict[str, int], in_features: int, dtype: torch.dtype):
        super().__init__()
        self.offsets, off = {}, 0
        for name, n in sections.items():
            self.offsets[name] = (off, n)
            off += n
        self.weight = _param(off, in_features, dtype=dtype)

    def section(self, name: str) -> torch.Tensor:
        off, n = self.offsets[name]
        return self.weight[off:off + n]

    def starts(self, *names: str):
        return [self.offsets[n][0] for n in names]

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return F.linear(x, self.weight)


class WindowAttention(nn.Module):
    """Grouped-query attention over a sliding window with kept first tokens, q and k normed over the whole projection, no
    positions in the scores, sigmoid output gate."""

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.spec = ops.WindowSpec(cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"], cfg["mask"]["size"], cfg["mask"]["keep_first"], float(cfg["scale"]))
        s = self.spec
        self.width, self.eps = width, eps
        self.qkvg = PackedLinear({"q": s.heads * s.dim, "k": s.kv_heads * s.dim, "v": s.kv_heads * s.vdim, "g": s.heads * s.vdim}, width, dtype)
        self.q_norm, self.k_norm = _param(s.heads * s.dim, dtype=torch.float32), _param(s.kv_heads * s.dim, dtype=torch.float32)
        self.o = PackedLinear({"o": width}, s.heads * s.vdim, dtype)

    def tensors(self) -> Dict[str, torch.Tensor]:
        """Checkpoint name (below the mixer) -> where it goes."""
        out = {n: self.qkvg.section(n) for n in "qkvg"}
        out.update({"q.norm": self.q_norm, "k.norm": self.k_norm, "o": self.o.weight})
        return out

    def forward(self, x, xh, state, batch):
        proj = self.qkvg(xh[:, :self.width])
        y = ops.window_attention(proj, self.qkvg.starts("q", "k", "v", "g"), self.q_norm, self.k_norm, self.eps, self.spec, state, batch)
        return self.o(y)


class MLSTM(nn.Module):
    """Matrix memory with exponential, soft-capped gates in log space; head norm and sigmoid output gate behind it."""

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.spec = ops.MlstmSpec(cfg["heads"], cfg["dim"], cfg["vdim"], float(cfg["gate_cap"]))
        s = self.spec
        self.width, self.eps = width, eps
        self.qkvg = PackedLinear({"q": s.heads * s.dim, "k": s.heads * s.dim, "v": s.heads * s.vdim, "g": s.heads * s.vdim}, width, dtype)
        self.gates = PackedLinear({"i": s.heads, "f": s.heads}, ops.padded(width), dtype)      # fp32 products: trimkv_linear_f32
        self.i_bias, self.f_bias = _param(s.heads, dtype=torch.float32), _param(s.heads, dtype=torch.float32)
        self.head_norm = _param(s.heads * s.vdim, dtype=torch.float32)
        self.o = PackedLinear({"o": width}, s.heads * s.vdim, dtype)

    def tensors(self) -> Dict[str, torch.Tensor]:
        out = {n: self.qkvg.section(n) for n in "qkvg"}
        out.update({n: self.gates.section(n)[:, :self.width] for n in "if"})
        out.update({"i.b": self.i_bias, "f.b": self.f_bias, "norm": self.head_norm, "o": self.o.weight})
        return out

    def forward(self, x, xh, state, batch):
        proj = self.qkvg(xh[:, :self.width])
        gates = ops.linear_f32(x, self.gates.weight)
        y = ops.mlstm(proj, self.qkvg.starts("q", "k", "v", "g"), gates, self.i_bias, self.f_bias, self.head_norm, self.eps, self.spec, state, batch)
        return self.o(y)


class ExpertMatrix:
    """Where one expert's [n, k] matrix of a checkpoint goes: its blocks in the packed stack (padding stays zero)."""

    def __init__(self, packed: torch.Tensor, n: int, k: int):
        self.packed, self.shape = packed, (n, k)
        self.device, self.dtype = packed.device, packed.dtype

    def dim(self) -> int:
        return 2

    def copy_(self, src: torch.Tensor) -> None:
        full = torch.zeros(self.packed.shape[0] * 32, self.packed.shape[1] * 16, dtype=self.dtype, device=self.device)
        full[:self.shape[0], :self.shape[1]] = src
        self.packed.copy_(ops.pack_matrix(full))

    def value(self) -> torch.Tensor:
        return ops.unpack_matrix(self.packed)[:self.shape[0], :self.shape[1]]


class RoutedExperts(nn.Module):
    """Squared-ReLU experts behind a grouped sigmoid router.  ``forward`` returns the chosen experts' outputs and their
    weights: the weighted sum is taken by whoever adds them to the residual stream."""

    def __init__(self, cfg: dict, width: int, dtype: torch.dtype):
        super().__init__()
        r, ff = cfg["router"], cfg["expert"]["ff"]
        groups = r.get("groups") or {"count": 1, "keep": 1}
        self.spec = ops.RouterSpec(r["experts"], r["top"], groups["count"], groups["keep"])
        self.width, self.ff = width, ff
        wp, fp = ops.padded(width), ops.padded(ff)
        self.router = _param(self.spec.experts, wp, dtype=dtype)
        self.correction = _param(self.spec.experts, dtype=torch.float32)
        self.up = _param(self.spec.experts, fp // 32, wp // 16, 2, 32, 8, dtype=dtype)       # packed, see trimkv_moe_gemm
        self.down = _param(self.spec.experts, wp // 32, fp // 16, 2, 32, 8, dtype=dtype)

    def tensors(self) -> Dict[str, torch.Tensor]:
        out = {"router": self.router[:, :self.width], "correction": self.correction}
        for e in range(self.spec.experts):
            out[f"e{e}.up"], out[f"e{e}.down"] = ExpertMatrix(self.up[e], self.ff, self.width), ExpertMatrix(self.down[e], self.width, self.ff)
        return out

    def forward(self, x, xh):
        ids, weights = ops.route(ops.linear_f32(x, self.router), self.correction, self.spec)
        return ops.experts(xh, ids, self.up, self.down, self.width), weights


MIXERS = {"attention": WindowAttention, "mlstm": MLSTM}
FEED_FORWARDS = {"moe": RoutedExperts}


class HybridLayer(nn.Module):
    def __init__(self, layer: dict, width: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.eps = eps
        self.mix = MIXERS[layer["type"]](layer["mixer"], width, eps, dtype)
        self.norm1 = _param(width, dtype=torch.float32)
        self.mlp = self.norm2 = None
        if layer.get("mlp") is not None:
            self.mlp = FEED_FORWARDS[layer["mlp"]["kind"]](layer["mlp"], width, dtype)
            self.norm2 = _param(width, dtype=torch.float32)

    def tensors(self) -> Dict[str, torch.Tensor]:
        out = {"norm1": self.norm1}
        out.update({f"mix.{k}": v for k, v in self.mix.tensors().items()})
        if self.mlp is not None:
            out["norm2"] = self.norm2
            out.update({f"mlp.{k}": v for k, v in self.mlp.tensors().items()})
        return out

    def forward(self, x, xh, state, batch):
        """Advances the stream (x fp32 and its copy xh in the matrices' dtype) in place."""
        src = x if xh is None else xh
        ops.residual_norm(x, xh, self.mix(x, src, state, batch), self.norm1, self.eps)
        if self.mlp is not None:
            y, weights = self.mlp(x, src)
            ops.residual_norm(x, xh, y, self.norm2, self.eps, weights)


class HybridModel(nn.Module):
    def __init__(self, config, dtype: torch.dtype):
        super().__init__()
        self.config, self.dtype = config, dtype
        self.embed = _param(config.vocab_size, config.hidden_size, dtype=dtype)
        self.layers = nn.ModuleList([HybridLayer(l, config.hidden_size, config.norm_eps, dtype) for l in config.layers])
        self.norm = _param(config.hidden_size, dtype=torch.float32)

    def new_cache(self, num_slots: int = 0) -> HybridCache:
        return HybridCache([l.mix.spec for l in self.layers], self.dtype, self.embed.device, num_slots)

    def forward(self, ids: torch.Tensor, cache: HybridCache, batch: ops.PackedBatch, layers_out: Optional[List[torch.Tensor]] = None):
        """The fp32 residual stream [T, width padded] behind the last layer; ``layers_out`` receives a copy behind every layer."""
        x, xh = ops.embed_scaled(ids, self.embed, self.config.embedding_scale, ops.padded(self.config.hidden_size))
        for layer, state in zip(self.layers, cache.layers_state):
            layer(x, xh, state, batch)
            if layers_out is not None:
                layers_out.append(x[:, :self.config.hidden_size].clone())
        cache.advance(batch)
        return x


class HybridForCausalLM(GreedyGeneration, nn.Module):
    """Model, tied head and step function.  ``config_cls`` reads config.json; checkpoint names come from ``tensors``."""
    config_cls = None

    def __init__(self, config, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{type(self).__name__} runs in bfloat16 or float32, not {dtype}")
        self.config = config
        self.model = HybridModel(config, dtype)

    @property
    def device(self) -> torch.device:
        return self.model.embed.device

    def new_cache(self, num_slots: int = 0) -> HybridCache:
        return self.model.new_cache(num_slots)

    # ---- weights ----------------------------------------------------------------------------------
    def tensors(self) -> Dict[str, torch.Tensor]:
        """Checkpoint name -> the (part of a) parameter it fills (has ``shape`` and ``copy_``)."""
        out = {"embed": self.model.embed, "final.norm": self.model.norm}
        for i, layer in enumerate(self.model.layers):
            out.update({f"l{i}.{k}": v for k, v in layer.tensors().items()})
        return out

    @torch.no_grad()
    def load_tensors(self, state: Dict[str, torch.Tensor]) -> None:
        want = self.tensors()
        missing, extra = sorted(set(want) - set(state)), sorted(set(state) - set(want))
        if missing or extra:
            raise ValueError(f"checkpoint does not fit the configuration: missing {missing[:4]}, unexpected {extra[:4]}")
        for name, dst in want.items():
            if tuple(state[name].shape) != tuple(dst.shape):
                raise ValueError(f"{name}: checkpoint has shape {tuple(state[name].shape)}, the configuration {tuple(dst.shape)}")
            dst.copy_(state[name])

    @torch.no_grad()
    def randomize(self, seed: int = 0) -> "HybridForCausalLM":
        """Random weights of sensible scale (there is no checkpoint to fetch): matrices with unit gain, norms of one."""
        gen = torch.Generator(device=self.device).manual_seed(seed)
        for name, t in self.tensors().items():
            if t.dim() > 1:
                # filled a slice at a time: expert stacks can be tens of GB
                t.copy_(torch.randn(t.shape, generator=gen, device=t.device, dtype=torch.float32) * (1.0 if name == "embed" else t.shape[-1] ** -0.5))
            elif name.endswith("norm") or "norm" in name.rsplit(".", 1)[-1]:
                t.fill_(1.0)
        return self

    @classmethod
    def from_pretrained(cls, path: str, torch_dtype: Optional[torch.dtype] = torch.bfloat16, **kwargs) -> "HybridForCausalLM":
        """A local directory with config.json and ``*.safetensors``; keyword arguments override configuration fields."""
        from .registry import load_checkpoint_tensors, read_config
        config = cls.config_cls.from_dict(read_config(path), **kwargs)
        model = cls(config, torch.bfloat16 if torch_dtype is None else torch_dtype)
        model.load_tensors(load_checkpoint_tensors(path))
        return model.eval()

    # ---- the step -----------------------------------------------------------------------------------
    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor, past_key_values: Optional[HybridCache] = None, lengths: Optional[Sequence[int]] = None,
                slots: Optional[Sequence[int]] = None, logits_to_keep: int = 0, rows: Optional[torch.Tensor] = None,
                layers_out: Optional[List[torch.Tensor]] = None):
        """One step over any number of sequences, all at their first token or all going on.

        ``input_ids``: [B, S] (with ``lengths``: padded on the right, padding is dropped before anything is computed) or the
        packed tokens [sum of lengths].  ``slots``: the cache slots of the sequences; by default all active ones, and new
        slots for a cache that holds none.  ``rows``: packed positions whose logits are wanted ([n, vocab] comes back);
        ``logits_to_keep`` = n: the last n of every sequence ([B, n, vocab]); neither: all ([B, S, vocab], or packed when
        the lengths differ)."""
        if not input_ids.is_cuda:
            raise _lib.TrimKVLibraryError(f"input_ids is on {input_ids.device}: the hybrid decoders run on the GPU only (no CPU path)")
        if input_ids.dim() == 2:
            B, S = input_ids.shape
            lengths = [S] * B if lengths is None else [int(n) for n in lengths]
            if len(lengths) != B or max(lengths) > S:
                raise ValueError(f"lengths {lengths} do not fit input_ids of shape {(B, S)}")
            packed = input_ids.reshape(-1) if min(lengths) == S else torch.cat([input_ids[b, :n] for b, n in enumerate(lengths)])
        else:
            if lengths is None:
                raise ValueError("packed input_ids need lengths")
            packed, B = input_ids, len(lengths)
            if sum(lengths) != packed.numel():
                raise ValueError(f"lengths {list(lengths)} do not add up to {packed.numel()} tokens")
        cache = self.new_cache(B) if past_key_values is None else past_key_values
        if slots is None and not cache.active:
            cache.allocate(B)
        batch = cache.batch(lengths, slots)
        x = self.model(packed.contiguous(), cache, batch, layers_out)
        keep = int(logits_to_keep)
        if rows is None and keep and batch.max_len > 1:
            if keep > min(batch.lengths):
                raise ValueError(f"logits_to_keep {keep} exceeds the shortest sequence of the step")
            ends, at = [], 0
            for n in batch.lengths:
                at += n
                ends += range(at - keep, at)
            rows = torch.tensor(ends, device=x.device)
            shape = (B, keep)
        else:
            shape = (-1,) if rows is not None or min(batch.lengths) != batch.max_len else (B, batch.max_len)
        h = ops.rms_rows(x, rows, self.model.norm, self.config.norm_eps, self.model.dtype)
        logits = F.linear(h, self.model.embed).float()
        return SimpleNamespace(logits=logits.view(*shape, logits.shape[-1]), past_key_values=cache)
