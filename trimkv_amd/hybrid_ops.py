"""Tensor-level calls into libtrimkv_hybrid.so (``include/trimkv_hybrid.h``): what the hybrid decoders are made of.

Activations and matrices are bf16 or fp32 (``dtype`` of the tensors decides), everything the header calls fp32 is fp32 in
both.  There is no CPU path and no torch fallback.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Sequence, Tuple

import torch

from . import _lib

PAD = 64     # widths of activations that enter grouped products are padded to this


def padded(n: int, to: int = PAD) -> int:
    return (n + to - 1) // to * to


def _check(rc: int, what: str) -> None:
    _lib.check_hybrid(rc, what)


def _require(dtype: torch.dtype, *tensors: Optional[torch.Tensor]) -> None:
    for t in tensors:
        if t is None:
            continue
        if not t.is_cuda:
            raise _lib.TrimKVLibraryError(f"tensor on {t.device}: the hybrid decoders run on the GPU only (no CPU path)")
        if t.dtype != dtype:
            raise _lib.TrimKVLibraryError(f"expected {dtype}, got {t.dtype}")
        if t.stride(-1) != 1:
            raise _lib.TrimKVLibraryError("rows must be contiguous")


@dataclass
class PackedBatch:
    """The sequences of one step, packed: sequence b owns tokens ``cu[b] : cu[b + 1]`` and cache slot ``slots[b]``."""
    lengths: Tuple[int, ...]
    slots: Tuple[int, ...]
    cu_dev: torch.Tensor
    slots_dev: torch.Tensor
    seen_dev: torch.Tensor       # [num_slots, 2]: tokens and steps before this step
    num_slots: int

    @property
    def batch(self) -> int:
        return len(self.lengths)

    @property
    def tokens(self) -> int:
        return sum(self.lengths)

    @property
    def max_len(self) -> int:
        return max(self.lengths)

    @property
    def decode(self) -> bool:
        return self.max_len == 1


def embed_scaled(ids: torch.Tensor, table: torch.Tensor, scale: float, stride: int):
    """fp32 rows [T, stride] of ``table[ids] * scale`` (zeros behind the width) and the same in the table's dtype (None for fp32)."""
    _require(table.dtype, table)
    _require(torch.int64, ids)
    T, (V, W) = ids.numel(), table.shape
    x = torch.empty(T, stride, dtype=torch.float32, device=ids.device)
    xh = None if table.dtype == torch.float32 else torch.empty(T, stride, dtype=table.dtype, device=ids.device)
    _check(_lib.load_hybrid().trimkv_embed_scaled(ids.data_ptr(), table.data_ptr(), scale, x.data_ptr(), _lib.ptr(xh), T, V, W, stride,
                                                  _lib.dtype_code(table.dtype), _lib.current_stream(ids.device)), "trimkv_embed_scaled")
    return x, xh


def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """fp32 ``x @ w.T`` for a narrow w [n, k] (fp32 products and sums whatever w's dtype)."""
    _require(torch.float32, x)
    _require(w.dtype, w)
    out = torch.empty(x.shape[0], w.shape[0], dtype=torch.float32, device=x.device)
    _check(_lib.load_hybrid().trimkv_linear_f32(x.data_ptr(), x.stride(0), w.data_ptr(), w.stride(0), out.data_ptr(), x.shape[0], w.shape[0], w.shape[1],
                                                _lib.dtype_code(w.dtype), _lib.current_stream(x.device)), "trimkv_linear_f32")
    return out


def residual_norm(x: torch.Tensor, xh: Optional[torch.Tensor], y: torch.Tensor, w: torch.Tensor, eps: float,
                  y_weight: Optional[torch.Tensor] = None) -> None:
    """In place: ``x += w * rms(y)`` and ``xh = x``; with ``y_weight`` [T, top], y holds top rows per token to be summed with those weights."""
    _require(y.dtype, y, xh)
    _require(torch.float32, x, w, y_weight)
    _check(_lib.load_hybrid().trimkv_residual_norm(y.data_ptr(), y.stride(0), _lib.ptr(y_weight), 1 if y_weight is None else y_weight.shape[1],
                                                   x.data_ptr(), w.data_ptr(), _lib.ptr(xh), x.shape[0], w.shape[0], x.stride(0), eps,
                                                   _lib.dtype_code(y.dtype), _lib.current_stream(x.device)), "trimkv_residual_norm")


def rms_rows(x: torch.Tensor, rows: Optional[torch.Tensor], w: torch.Tensor, eps: float, dtype: torch.dtype) -> torch.Tensor:
    _require(torch.float32, x, w)
    count = x.shape[0] if rows is None else rows.numel()
    out = torch.empty(count, w.shape[0], dtype=dtype, device=x.device)
    _check(_lib.load_hybrid().trimkv_rms_rows(x.data_ptr(), x.stride(0), _lib.ptr(rows), w.data_ptr(), out.data_ptr(), count, w.shape[0], eps,
                                              _lib.dtype_code(dtype), _lib.current_stream(x.device)), "trimkv_rms_rows")
    return out


@dataclass(frozen=True)
class WindowSpec:
    """Sizes of one windowed attention layer; ``rows`` cache rows per (sequence, KV head) whatever the length."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    window: int
    keep_first: int
    scale: float

    @property
    def rows(self) -> int:
        return self.keep_first + self.window

    @property
    def dim_stride(self) -> int:
        return padded(self.dim, 8)

    @property
    def vdim_stride(self) -> int:
        return padded(self.vdim, 8)

    def state_shapes(self, slots: int, dtype: torch.dtype):
        return {"k": ((slots, self.kv_heads, self.rows, self.dim_stride), dtype), "v": ((slots, self.kv_heads, self.rows, self.vdim_stride), dtype)}


@dataclass(frozen=True)
class MlstmSpec:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def state_shapes(self, slots: int, dtype: torch.dtype):
        return {"S": ((slots, self.heads, self.dim, self.vdim), torch.float32), "nm": ((2, slots, self.heads, self.dim + 1), torch.float32)}


def window_attention(proj: torch.Tensor, offsets: Sequence[int], q_norm: torch.Tensor, k_norm: torch.Tensor, eps: float, spec: WindowSpec,
                     ring: dict, batch: PackedBatch) -> torch.Tensor:
    """proj [T, q|k|v|gate at ``offsets``] -> gated attention output [T, heads * vdim]; the batch's tokens end up in the ring."""
    dt = proj.dtype
    _require(dt, proj, ring["k"], ring["v"])
    _require(torch.float32, q_norm, k_norm)
    lib, st, code = _lib.load_hybrid(), _lib.current_stream(proj.device), _lib.dtype_code(dt)
    T, s = proj.shape[0], spec
    qo, ko, vo, go = offsets
    q = torch.empty(T, s.heads, s.dim_stride, dtype=dt, device=proj.device)
    out = torch.empty(T, s.heads * s.vdim, dtype=dt, device=proj.device)
    gate = proj.data_ptr() + go * proj.element_size()
    common = (proj.data_ptr(), proj.stride(0), qo, ko, vo, q_norm.data_ptr(), k_norm.data_ptr(), eps, s.heads, s.kv_heads, s.dim, s.vdim, s.dim_stride, s.vdim_stride)
    slots, seen = batch.slots_dev.data_ptr(), batch.seen_dev.data_ptr()
    rk, rv = ring["k"].data_ptr(), ring["v"].data_ptr()
    if batch.decode:
        _check(lib.trimkv_qkv_norm(*common, q.data_ptr(), rk, rv, slots, seen, s.keep_first, s.window, T, code, st), "trimkv_qkv_norm")
        splits = lib.trimkv_window_decode_splits(batch.batch, s.kv_heads, s.rows)
        ws = torch.empty(T * s.heads * splits * (s.vdim + 2), dtype=torch.float32, device=proj.device) if splits > 1 else None
        _check(lib.trimkv_window_decode(q.data_ptr(), rk, rv, slots, seen, gate, proj.stride(0), out.data_ptr(), T, s.heads, s.kv_heads, s.dim, s.vdim,
                                        s.dim_stride, s.vdim_stride, s.keep_first, s.window, s.scale, splits, _lib.ptr(ws), code, st), "trimkv_window_decode")
        return out
    k = torch.empty(T, s.kv_heads, s.dim_stride, dtype=dt, device=proj.device)
    v = torch.empty(T, s.kv_heads, s.vdim_stride, dtype=dt, device=proj.device)
    _check(lib.trimkv_qkv_norm(*common, q.data_ptr(), k.data_ptr(), v.data_ptr(), None, None, 0, 0, T, code, st), "trimkv_qkv_norm")
    cu = batch.cu_dev.data_ptr()
    _check(lib.trimkv_window_prefill(q.data_ptr(), k.data_ptr(), v.data_ptr(), rk, rv, cu, slots, seen, gate, proj.stride(0), out.data_ptr(),
                                     batch.batch, batch.max_len, s.heads, s.kv_heads, s.dim, s.vdim, s.dim_stride, s.vdim_stride,
                                     s.keep_first, s.window, s.scale, code, st), "trimkv_window_prefill")
    _check(lib.trimkv_ring_store(k.data_ptr(), v.data_ptr(), cu, slots, seen, rk, rv, batch.batch, batch.max_len, s.kv_heads, s.dim_stride, s.vdim_stride,
                                 s.keep_first, s.window, code, st), "trimkv_ring_store")
    return out


def mlstm(proj: torch.Tensor, offsets: Sequence[int], gates: torch.Tensor, i_bias: torch.Tensor, f_bias: torch.Tensor, head_norm: torch.Tensor, eps: float,
          spec: MlstmSpec, state: dict, batch: PackedBatch) -> torch.Tensor:
    """proj [T, q|k|v|gate at ``offsets``], gates fp32 [T, 2 heads] -> normed and gated output [T, heads * vdim]; advances the state."""
    _require(proj.dtype, proj)
    _require(torch.float32, gates, i_bias, f_bias, head_norm, state["S"], state["nm"])
    lib, st, code = _lib.load_hybrid(), _lib.current_stream(proj.device), _lib.dtype_code(proj.dtype)
    T, s = proj.shape[0], spec
    qo, ko, vo, go = offsets
    o = torch.empty(T, s.heads, s.vdim, dtype=proj.dtype, device=proj.device)
    out = torch.empty(T, s.heads * s.vdim, dtype=proj.dtype, device=proj.device)
    need = lib.trimkv_mlstm_workspace(batch.batch, batch.max_len, s.heads, s.dim, s.vdim, code)
    ws = torch.empty(need, dtype=torch.float32, device=proj.device) if need else None
    _check(lib.trimkv_mlstm(proj.data_ptr(), proj.stride(0), qo, ko, vo, gates.data_ptr(), i_bias.data_ptr(), f_bias.data_ptr(), s.gate_cap,
                            state["S"].data_ptr(), state["nm"].data_ptr(), batch.cu_dev.data_ptr(), batch.slots_dev.data_ptr(), batch.seen_dev.data_ptr(),
                            o.data_ptr(), batch.batch, batch.max_len, s.heads, s.dim, s.vdim, batch.num_slots, s.dim ** -0.5, _lib.ptr(ws), code, st), "trimkv_mlstm")
    _check(lib.trimkv_head_norm_gate(o.data_ptr(), proj.data_ptr() + go * proj.element_size(), proj.stride(0), head_norm.data_ptr(), out.data_ptr(),
                                     T, s.heads, s.vdim, eps, code, st), "trimkv_head_norm_gate")
    return out


@dataclass(frozen=True)
class RouterSpec:
    """Sigmoid router: ``top`` of ``experts``, chosen inside the ``keep`` best of ``groups`` groups of neighbours."""
    experts: int
    top: int
    groups: int
    keep: int


def route(logits: torch.Tensor, correction: torch.Tensor, spec: RouterSpec):
    _require(torch.float32, logits, correction)
    T = logits.shape[0]
    ids = torch.empty(T, spec.top, dtype=torch.int32, device=logits.device)
    weights = torch.empty(T, spec.top, dtype=torch.float32, device=logits.device)
    _check(_lib.load_hybrid().trimkv_moe_route(logits.data_ptr(), correction.data_ptr(), ids.data_ptr(), weights.data_ptr(), T, spec.experts, spec.top,
                                               spec.groups, spec.keep, _lib.current_stream(logits.device)), "trimkv_moe_route")
    return ids, weights


def pack_matrix(w: torch.Tensor) -> torch.Tensor:
    """[..., n, k] (multiples of 64) in the blocks trimkv_moe_gemm reads, [..., n / 32, k / 16, 2, 32, 8]."""
    *lead, n, k = w.shape
    return w.reshape(*lead, n // 32, 32, k // 16, 2, 8).movedim(-4, -2)


def unpack_matrix(p: torch.Tensor) -> torch.Tensor:
    *lead, nb, kb, _, _, _ = p.shape
    return p.movedim(-2, -4).reshape(*lead, nb * 32, kb * 16)


def experts(x: torch.Tensor, ids: torch.Tensor, up: torch.Tensor, down: torch.Tensor, width: int) -> torch.Tensor:
    """Rows x [T, k padded], expert ids [T, top], packed matrices up [E, ff, width] and down [E, width, ff] (``pack_matrix`` of
    the zero-padded ones) -> [T * top, width]: ``down_e relu(up_e x)^2`` of every (token, choice)."""
    _require(up.dtype, x, up, down)
    E, ffp, wp = up.shape[0], up.shape[1] * 32, up.shape[2] * 16
    T, top = ids.shape
    M, dev, lib, st, code = T * top, x.device, _lib.load_hybrid(), _lib.current_stream(x.device), _lib.dtype_code(up.dtype)
    # rows per expert: many -> tiles of the matrix-bound kernel, a few -> the weights stream past them
    tile = 16 if up.dtype == torch.float32 else 256 if M >= 96 * E else 32
    most = M if M < E else (M - E) // tile + E
    order = torch.empty(M, dtype=torch.int32, device=dev)
    offsets = torch.empty(E + 1, dtype=torch.int32, device=dev)
    tiles = torch.empty(1 + 2 * most, dtype=torch.int32, device=dev)
    _check(lib.trimkv_moe_plan(ids.data_ptr(), M, E, tile, order.data_ptr(), offsets.data_ptr(), tiles.data_ptr(), st), "trimkv_moe_plan")
    h = torch.empty(M, ffp, dtype=up.dtype, device=dev)
    y = torch.empty(M, width, dtype=up.dtype, device=dev)
    plan = (order.data_ptr(), offsets.data_ptr(), tiles.data_ptr(), M, E, tile, top)
    _check(lib.trimkv_moe_gemm(x.data_ptr(), x.stride(0), up.data_ptr(), h.data_ptr(), ffp, *plan, ffp, ffp, wp, 1, code, st), "trimkv_moe_gemm")
    _check(lib.trimkv_moe_gemm(h.data_ptr(), ffp, down.data_ptr(), y.data_ptr(), width, *plan, width, wp, ffp, 0, code, st), "trimkv_moe_gemm")
    return y


def advance(batch: PackedBatch) -> None:
    _check(_lib.load_hybrid().trimkv_advance(batch.seen_dev.data_ptr(), batch.slots_dev.data_ptr(), batch.cu_dev.data_ptr(), batch.batch,
                                             _lib.current_stream(batch.seen_dev.device)), "trimkv_advance")
