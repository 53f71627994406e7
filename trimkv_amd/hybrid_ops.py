"""Tensor-level calls into libtrimkv_hybrid.so, libtrimkv_mlstm.so and libtrimkv_moe.so (``include/trimkv_hybrid.h``): what the
hybrid decoders are made of.

Activations and matrices are bf16 or fp32 (``dtype`` of the tensors decides), everything the header calls fp32 is fp32 in
both.  There is no CPU path and no torch fallback.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, Optional, Sequence, Tuple

import torch

from . import _lib

PAD = 64     # widths of activations that enter grouped products are padded to this


def padded(n: int, to: int = PAD) -> int:
    return (n + to - 1) // to * to


def _check(rc: int, what: str, library: str = "hybrid") -> None:
    _lib.check_hybrid(rc, what, library)


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
    angles: Dict = field(default_factory=dict)      # rotation -> table of this step's positions (``rotary_table``)

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


def embed_scaled(ids: torch.Tensor, table: torch.Tensor, scale: float, stride: int, norm: Optional[torch.Tensor] = None, eps: float = 0.0,
                 add_to: Optional[Tuple[torch.Tensor, Optional[torch.Tensor]]] = None):
    """fp32 rows x [T, stride] of ``table[ids] * scale`` (zeros behind the width) and xh: the same in the table's dtype (None
    for fp32), or ``norm * rms(x)`` in that dtype.  ``add_to`` = (x, xh) of an earlier call: added to that x in place."""
    _require(table.dtype, table)
    _require(torch.int64, ids)
    _require(torch.float32, norm)
    T, (V, W) = ids.numel(), table.shape
    if add_to is None:
        x = torch.empty(T, stride, dtype=torch.float32, device=ids.device)
        xh = None if table.dtype == torch.float32 and norm is None else torch.empty(T, stride, dtype=table.dtype, device=ids.device)
    else:
        x, xh = add_to
        _require(torch.float32, x)
        _require(table.dtype, xh)
    _check(_lib.load_hybrid().trimkv_embed_scaled(ids.data_ptr(), table.data_ptr(), scale, x.data_ptr(), _lib.ptr(xh), _lib.ptr(norm), eps, int(add_to is not None),
                                                  T, V, W, stride, _lib.dtype_code(table.dtype), _lib.current_stream(ids.device)), "trimkv_embed_scaled")
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
                  y_weight: Optional[torch.Tensor] = None, mult: float = 1.0, next_norm: Optional[torch.Tensor] = None) -> None:
    """In place: ``x += mult * w * rms(y)`` and ``xh = x`` or ``xh = next_norm * rms(x)``; with ``y_weight`` [T, top], y holds top
    rows per token to be summed with those weights."""
    _require(y.dtype, y, xh)
    _require(torch.float32, x, w, y_weight, next_norm)
    _check(_lib.load_hybrid().trimkv_residual_norm(y.data_ptr(), y.stride(0), _lib.ptr(y_weight), 1 if y_weight is None else y_weight.shape[1],
                                                   x.data_ptr(), w.data_ptr(), mult, _lib.ptr(xh), _lib.ptr(next_norm), x.shape[0], w.shape[0], x.stride(0), eps,
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
    """Sizes of one windowed attention layer; ``rows`` cache rows per (sequence, KV head) whatever the length.  ``head_gate``: one
    output gate per head instead of one per value; ``sink``: one more term, exp(0), in the softmax denominator."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    window: int
    keep_first: int
    scale: float
    head_gate: bool = False
    sink: bool = False

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


@dataclass(frozen=True)
class RotarySpec:
    """Rotary positions on the first ``dims`` features of a head, pairs (i, i + dims / 2): pair i turns by position *
    base^(-2 i / dims) / factor."""
    dims: int
    base: float
    factor: float = 1.0

    def frequencies(self) -> torch.Tensor:
        return torch.tensor([self.base ** (-2.0 * i / self.dims) / self.factor for i in range(self.dims // 2)], dtype=torch.float64)


def rotary_table(spec: RotarySpec, freq: torch.Tensor, batch: PackedBatch) -> torch.Tensor:
    """fp32 cosines and sines [T, dims] of the positions of this step, computed once for all layers that turn alike."""
    if spec not in batch.angles:
        _require(torch.float64, freq)
        table = torch.empty(batch.tokens, spec.dims, dtype=torch.float32, device=freq.device)
        _check(_lib.load_hybrid().trimkv_rotary_table(freq.data_ptr(), batch.cu_dev.data_ptr(), batch.slots_dev.data_ptr(), batch.seen_dev.data_ptr(), table.data_ptr(),
                                                      batch.batch, batch.max_len, spec.dims, _lib.current_stream(freq.device)), "trimkv_rotary_table")
        batch.angles[spec] = table
    return batch.angles[spec]


@dataclass
class HeadForm:
    """What happens to the heads of q and k between projection and scores when they are normed one by one: ``bias`` (fp32, a
    number per column of the projection; v's is added too), then the norm, then the rotation by ``table``."""
    bias: Optional[torch.Tensor] = None
    table: Optional[torch.Tensor] = None


def window_attention(proj: torch.Tensor, offsets: Sequence[int], q_norm: Optional[torch.Tensor], k_norm: Optional[torch.Tensor], eps: float, spec: WindowSpec,
                     ring: dict, batch: PackedBatch, heads: Optional[HeadForm] = None) -> torch.Tensor:
    """proj [T, q|k|v|gate at ``offsets``] -> gated attention output [T, heads * vdim]; the batch's tokens end up in the ring.
    q and k are normed over all their heads at once (weights of those sizes) or, with ``heads``, as it says (weights [dim])."""
    dt = proj.dtype
    _require(dt, proj, ring["k"], ring["v"])
    _require(torch.float32, q_norm, k_norm)
    if heads is not None:
        _require(torch.float32, heads.bias, heads.table)
    lib, st, code = _lib.load_hybrid(), _lib.current_stream(proj.device), _lib.dtype_code(dt)
    T, s = proj.shape[0], spec
    qo, ko, vo, go = offsets
    q = torch.empty(T, s.heads, s.dim_stride, dtype=dt, device=proj.device)
    out = torch.empty(T, s.heads * s.vdim, dtype=dt, device=proj.device)
    gate = proj.data_ptr() + go * proj.element_size()
    sizes = (s.heads, s.kv_heads, s.dim, s.vdim, s.dim_stride, s.vdim_stride)
    if heads is None:
        place, what = lib.trimkv_qkv_norm, "trimkv_qkv_norm"
        common = (proj.data_ptr(), proj.stride(0), qo, ko, vo, q_norm.data_ptr(), k_norm.data_ptr(), eps, *sizes)
    else:
        place, what = lib.trimkv_qkv_heads, "trimkv_qkv_heads"
        common = (proj.data_ptr(), proj.stride(0), qo, ko, vo, _lib.ptr(heads.bias), _lib.ptr(q_norm), _lib.ptr(k_norm), eps, _lib.ptr(heads.table),
                  0 if heads.table is None else heads.table.shape[1], *sizes)
    slots, seen = batch.slots_dev.data_ptr(), batch.seen_dev.data_ptr()
    rk, rv = ring["k"].data_ptr(), ring["v"].data_ptr()
    if batch.decode:
        _check(place(*common, q.data_ptr(), rk, rv, slots, seen, s.keep_first, s.window, T, code, st), what)
        splits = lib.trimkv_window_decode_splits(batch.batch, s.kv_heads, s.rows)
        ws = torch.empty(T * s.heads * splits * (s.vdim + 2), dtype=torch.float32, device=proj.device) if splits > 1 else None
        _check(lib.trimkv_window_decode(q.data_ptr(), rk, rv, slots, seen, gate, proj.stride(0), out.data_ptr(), T, s.heads, s.kv_heads, s.dim, s.vdim,
                                        s.dim_stride, s.vdim_stride, s.keep_first, s.window, s.scale, int(s.head_gate), int(s.sink), splits, _lib.ptr(ws), code, st),
               "trimkv_window_decode")
        return out
    k = torch.empty(T, s.kv_heads, s.dim_stride, dtype=dt, device=proj.device)
    v = torch.empty(T, s.kv_heads, s.vdim_stride, dtype=dt, device=proj.device)
    _check(place(*common, q.data_ptr(), k.data_ptr(), v.data_ptr(), None, None, 0, 0, T, code, st), what)
    cu = batch.cu_dev.data_ptr()
    _check(lib.trimkv_window_prefill(q.data_ptr(), k.data_ptr(), v.data_ptr(), rk, rv, cu, slots, seen, gate, proj.stride(0), out.data_ptr(),
                                     batch.batch, batch.max_len, s.heads, s.kv_heads, s.dim, s.vdim, s.dim_stride, s.vdim_stride,
                                     s.keep_first, s.window, s.scale, int(s.head_gate), int(s.sink), code, st), "trimkv_window_prefill")
    _check(lib.trimkv_ring_store(k.data_ptr(), v.data_ptr(), cu, slots, seen, rk, rv, batch.batch, batch.max_len, s.kv_heads, s.dim_stride, s.vdim_stride,
                                 s.keep_first, s.window, code, st), "trimkv_ring_store")
    return out


def mlstm(proj: torch.Tensor, offsets: Sequence[int], gates: torch.Tensor, i_bias: torch.Tensor, f_bias: torch.Tensor, head_norm: torch.Tensor, eps: float,
          spec: MlstmSpec, state: dict, batch: PackedBatch) -> torch.Tensor:
    """proj [T, q|k|v|gate at ``offsets``], gates fp32 [T, 2 heads] -> normed and gated output [T, heads * vdim]; advances the state."""
    _require(proj.dtype, proj)
    _require(torch.float32, gates, i_bias, f_bias, head_norm, state["S"], state["nm"])
    lib, st, code = _lib.load_hybrid("mlstm"), _lib.current_stream(proj.device), _lib.dtype_code(proj.dtype)
    T, s = proj.shape[0], spec
    qo, ko, vo, go = offsets
    o = torch.empty(T, s.heads, s.vdim, dtype=proj.dtype, device=proj.device)
    out = torch.empty(T, s.heads * s.vdim, dtype=proj.dtype, device=proj.device)
    need = lib.trimkv_mlstm_workspace(batch.batch, batch.max_len, s.heads, s.dim, s.vdim, code)
    ws = torch.empty(need, dtype=torch.float32, device=proj.device) if need else None
    _check(lib.trimkv_mlstm(proj.data_ptr(), proj.stride(0), qo, ko, vo, gates.data_ptr(), i_bias.data_ptr(), f_bias.data_ptr(), s.gate_cap,
                            state["S"].data_ptr(), state["nm"].data_ptr(), batch.cu_dev.data_ptr(), batch.slots_dev.data_ptr(), batch.seen_dev.data_ptr(),
                            o.data_ptr(), batch.batch, batch.max_len, s.heads, s.dim, s.vdim, batch.num_slots, s.dim ** -0.5, _lib.ptr(ws), code, st), "trimkv_mlstm", "mlstm")
    _check(_lib.load_hybrid().trimkv_head_norm_gate(o.data_ptr(), proj.data_ptr() + go * proj.element_size(), proj.stride(0), head_norm.data_ptr(), out.data_ptr(),
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
    _check(_lib.load_hybrid("moe").trimkv_moe_route(logits.data_ptr(), correction.data_ptr(), ids.data_ptr(), weights.data_ptr(), T, spec.experts, spec.top,
                                               spec.groups, spec.keep, _lib.current_stream(logits.device)), "trimkv_moe_route", "moe")
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
    M, dev, lib, st, code = T * top, x.device, _lib.load_hybrid("moe"), _lib.current_stream(x.device), _lib.dtype_code(up.dtype)
    # rows per expert: many -> tiles of the matrix-bound kernel, a few -> the weights stream past them
    tile = 16 if up.dtype == torch.float32 else 256 if M >= 96 * E else 32
    most = M if M < E else (M - E) // tile + E
    order = torch.empty(M, dtype=torch.int32, device=dev)
    offsets = torch.empty(E + 1, dtype=torch.int32, device=dev)
    tiles = torch.empty(1 + 2 * most, dtype=torch.int32, device=dev)
    _check(lib.trimkv_moe_plan(ids.data_ptr(), M, E, tile, order.data_ptr(), offsets.data_ptr(), tiles.data_ptr(), st), "trimkv_moe_plan", "moe")
    h = torch.empty(M, ffp, dtype=up.dtype, device=dev)
    y = torch.empty(M, width, dtype=up.dtype, device=dev)
    plan = (order.data_ptr(), offsets.data_ptr(), tiles.data_ptr(), M, E, tile, top)
    _check(lib.trimkv_moe_gemm(x.data_ptr(), x.stride(0), up.data_ptr(), h.data_ptr(), ffp, *plan, ffp, ffp, wp, 1, code, st), "trimkv_moe_gemm", "moe")
    _check(lib.trimkv_moe_gemm(h.data_ptr(), ffp, down.data_ptr(), y.data_ptr(), width, *plan, width, wp, ffp, 0, code, st), "trimkv_moe_gemm", "moe")
    return y


def silu_gate(both: torch.Tensor, inter: int) -> torch.Tensor:
    """both [T, gate|up], ``inter`` columns each -> silu(gate) * up [T, inter]."""
    _require(both.dtype, both)
    out = torch.empty(both.shape[0], inter, dtype=both.dtype, device=both.device)
    _check(_lib.load_hybrid().trimkv_silu_gate(both.data_ptr(), both.data_ptr() + inter * both.element_size(), both.stride(0), out.data_ptr(), both.shape[0], inter,
                                               _lib.dtype_code(both.dtype), _lib.current_stream(both.device)), "trimkv_silu_gate")
    return out


def soft_cap(x: torch.Tensor, cap: float) -> torch.Tensor:
    """fp32 ``cap * tanh(x / cap)``."""
    x = x.contiguous()
    _require(x.dtype, x)
    out = torch.empty(x.shape, dtype=torch.float32, device=x.device)
    _check(_lib.load_hybrid().trimkv_soft_cap(x.data_ptr(), out.data_ptr(), x.numel(), cap, _lib.dtype_code(x.dtype), _lib.current_stream(x.device)), "trimkv_soft_cap")
    return out


def advance(batch: PackedBatch) -> None:
    _check(_lib.load_hybrid().trimkv_advance(batch.seen_dev.data_ptr(), batch.slots_dev.data_ptr(), batch.cu_dev.data_ptr(), batch.batch,
                                             _lib.current_stream(batch.seen_dev.device)), "trimkv_advance")
