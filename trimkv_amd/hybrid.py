"""Decoders whose layers mix windowed attention with recurrent layers, dense feed-forwards and routed experts, on the kernels
of libtrimkv_hybrid.so, libtrimkv_mlstm.so and libtrimkv_moe.so.

A layer is a mixer and, optionally, a feed-forward; both are looked up by kind (``MIXERS``, ``FEED_FORWARDS``) and bring
their sizes and variants as parameters, so another design of the same kind is another configuration (``HybridConfig``).  The
residual stream is fp32; the norms sit behind the sublayers, which read the stream itself (``x += norm(sublayer(x))``), or on
both sides of them.  A run of layers may be passed several times, each pass with a state of its own.  Matrices and activations
are bf16 or fp32 throughout; norm weights, biases and corrections are fp32.

Batches are packed: the tokens of unequal sequences lie one after the other, no padding is computed.  The same forward serves
prompts, portions of prompts and decode steps; what a sequence leaves behind is in a ``HybridCache``.
"""
from __future__ import annotations

from dataclasses import dataclass
from types import SimpleNamespace
from typing import Dict, List, NamedTuple, Optional, Sequence, Tuple

import torch
from torch import nn
import torch.nn.functional as F

from . import _lib, hybrid_ops as ops
from .generation import GreedyGeneration
from .hybrid_cache import HybridCache


class LayerRun(NamedTuple):
    """One execution of a layer; ``again``: a further pass begins with it, the embedding joins the stream in front of it."""
    index: int
    again: bool


_MIXER_KEYS = {"attention": ("heads", "kv_heads", "dim", "vdim", "scale", "mask"), "mlstm": ("heads", "dim", "vdim", "gate_cap")}


@dataclass
class HybridConfig:
    """What a hybrid decoder is made of.  ``layers``: entries with ``type``, ``mixer`` and ``mlp`` as the classes in ``MIXERS`` and
    ``FEED_FORWARDS`` take them.  ``norms``: "after" the sublayers or on "both" sides.  ``loop``: layers ``start`` .. ``stop`` - 1
    run ``times`` times in a row, and the embedding is added to the stream between two passes."""
    vocab_size: int
    hidden_size: int
    norm_eps: float
    layers: List[dict]
    architecture: str = ""
    embedding_scale: float = 1.0
    tied_head: bool = True
    norms: str = "after"
    residual_mult: float = 1.0
    loop: Optional[dict] = None
    logit_softcap: Optional[float] = None

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def layer_runs(self) -> List[LayerRun]:
        """The layers in the order of execution."""
        if not self.loop:
            return [LayerRun(i, False) for i in range(len(self.layers))]
        start, stop = self.loop["start"], self.loop["stop"]
        order = list(range(start)) + list(range(start, stop)) * self.loop["times"] + list(range(stop, len(self.layers)))
        entries = {start + n * (stop - start) for n in range(1, self.loop["times"])}
        return [LayerRun(i, n in entries) for n, i in enumerate(order)]

    def validate(self) -> None:
        if not self.layers:
            raise ValueError(f"a {self.architecture} model needs at least one layer")
        if self.norms not in ("after", "both"):
            raise ValueError(f"unknown placement of norms {self.norms!r}")
        if self.loop and not (0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers) and self.loop["times"] >= 1):
            raise ValueError(f"loop {self.loop} does not fit {len(self.layers)} layers")
        if self.logit_softcap is not None and not self.logit_softcap > 0:
            raise ValueError(f"logit_softcap must be positive, not {self.logit_softcap}")
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
                if m["mask"]["size"] < 1 or m["mask"].get("keep_first", 0) < 0:
                    raise ValueError(f"layer {i}: bad window {m['mask']}")
                rot = m.get("rot")
                if rot and (rot["dims"] % 2 or not 0 < rot["dims"] <= m["dim"] or not rot["base"] > 0 or not rot["scaling"]["factor"] > 0):
                    raise ValueError(f"layer {i}: bad rotation {rot} for heads of {m['dim']}")
            if mlp is not None:
                if mlp.get("kind") not in FEED_FORWARDS:
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r} (one of {sorted(FEED_FORWARDS)})")
                if mlp["kind"] == "dense" and mlp["ff"] < 1:
                    raise ValueError(f"layer {i}: bad feed-forward {mlp}")
                if mlp["kind"] == "moe":
                    r = mlp["router"]
                    g = r.get("groups") or {"count": 1, "keep": 1}
                    if r["experts"] % g["count"] or not 1 <= g["keep"] <= g["count"] or not 1 <= r["top"] <= g["keep"] * (r["experts"] // g["count"]):
                        raise ValueError(f"layer {i}: router {r} cannot choose {r['top']} experts")
            if self.norms == "both" and (MIXERS[kind].reads_stream or (mlp is not None and FEED_FORWARDS[mlp["kind"]].reads_stream)):
                raise ValueError(f"layer {i}: {kind} / {mlp and mlp['kind']} takes the fp32 stream itself and cannot follow a norm")


def _param(*shape, dtype) -> nn.Parameter:
    return nn.Parameter(torch.zeros(*shape, dtype=dtype), requires_grad=False)


class PackedLinear(nn.Module):
    """Several matrices over the same input as one weight; ``section(name)`` is the rows of one of them.  ``align``: rows of
    zeros bring the output to a multiple of that."""

    def __init__(self, sections: Dict[str, int], in_features: int, dtype: torch.dtype, align: int = 1):
        super().__init__()
        self.offsets, off = {}, 0
        for name, n in sections.items():
            self.offsets[name] = (off, n)
            off += n
        self.weight = _param(ops.padded(off, align), in_features, dtype=dtype)

    def section(self, name: str) -> torch.Tensor:
        off, n = self.offsets[name]
        return self.weight[off:off + n]

    def starts(self, *names: str):
        return [self.offsets[n][0] for n in names]

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return F.linear(x, self.weight)


class WindowAttention(nn.Module):
    """Grouped-query attention over a sliding window with kept first tokens and a sigmoid output gate.

    Variants, beside the sizes: ``qk_norm`` "projection" (all heads of q, or k, at once) or "head" (each by itself, one weight for
    all) or "none"; with the latter two also ``bias`` on q, k and v and ``rot``ary positions.  ``gate``: a number per "value" or per
    "head".  ``sink``: a score of 0 without a value in the softmax.  No rotation: no positions in the scores."""
    reads_stream, library = False, None

    def __init__(self, cfg: dict, width: int, eps: float, dtype: torch.dtype):
        super().__init__()
        norm, head_gate, rot = cfg.get("qk_norm", "projection"), cfg.get("gate", "value") == "head", cfg.get("rot")
        self.spec = ops.WindowSpec(cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"], cfg["mask"]["size"], cfg["mask"].get("keep_first", 0), float(cfg["scale"]),
                                   head_gate, bool(cfg.get("sink")))
        s = self.spec
        self.width, self.eps, self.by_head = width, eps, norm != "projection"
        if not self.by_head and (rot or cfg.get("bias")):
            raise ValueError("rotary positions and biases need heads that are normed one by one")
        self.qkvg = PackedLinear({"q": s.heads * s.dim, "k": s.kv_heads * s.dim, "v": s.kv_heads * s.vdim, "g": s.heads * (1 if head_gate else s.vdim)}, width, dtype, align=8)
        self.q_norm = self.k_norm = self.bias = self.rotation = None
        if norm != "none":
            self.q_norm, self.k_norm = (_param(s.dim if self.by_head else n * s.dim, dtype=torch.float32) for n in (s.heads, s.kv_heads))
        if cfg.get("bias"):
            self.bias = _param(self.qkvg.weight.shape[0], dtype=torch.float32)
        if rot:
            self.rotation = ops.RotarySpec(rot["dims"], float(rot["base"]), float(rot["scaling"]["factor"]))
            self.register_buffer("freq", self.rotation.frequencies(), persistent=False)
        self.o = PackedLinear({"o": width}, s.heads * s.vdim, dtype)

    def tensors(self) -> Dict[str, torch.Tensor]:
        """Checkpoint name (below the mixer) -> where it goes."""
        out = {n: self.qkvg.section(n) for n in "qkvg"}
        out["o"] = self.o.weight
        if self.q_norm is not None:
            out.update({"q.norm": self.q_norm, "k.norm": self.k_norm})
        if self.bias is not None:
            out.update({f"{n}.b": self.bias[off:off + size] for n, (off, size) in self.qkvg.offsets.items() if n != "g"})
        return out

    def forward(self, x, xh, state, batch):
        heads = None
        if self.by_head:
            heads = ops.HeadForm(self.bias, None if self.rotation is None else ops.rotary_table(self.rotation, self.freq, batch))
        proj = self.qkvg(xh[:, :self.width])
        y = ops.window_attention(proj, self.qkvg.starts("q", "k", "v", "g"), self.q_norm, self.k_norm, self.eps, self.spec, state, batch, heads)
        return self.o(y)


class MLSTM(nn.Module):
    """Matrix memory with exponential, soft-capped gates in log space; head norm and sigmoid output gate behind it."""
    reads_stream, library = True, "mlstm"

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
    reads_stream, library = True, "moe"

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


class DenseMLP(nn.Module):
    """``down (silu(gate h) * (up h))``, gate and up as one product."""
    reads_stream, library = False, None

    def __init__(self, cfg: dict, width: int, dtype: torch.dtype):
        super().__init__()
        self.width, self.ff = width, cfg["ff"]
        self.gate_up = PackedLinear({"gate": self.ff, "up": self.ff}, width, dtype)
        self.down = PackedLinear({"down": width}, self.ff, dtype)

    def tensors(self) -> Dict[str, torch.Tensor]:
        return {"gate": self.gate_up.section("gate"), "up": self.gate_up.section("up"), "down": self.down.weight}

    def forward(self, x, xh):
        return self.down(ops.silu_gate(self.gate_up(xh[:, :self.width]), self.ff)), None


MIXERS = {"attention": WindowAttention, "mlstm": MLSTM}
FEED_FORWARDS = {"moe": RoutedExperts, "dense": DenseMLP}


class HybridLayer(nn.Module):
    def __init__(self, layer: dict, config: HybridConfig, dtype: torch.dtype):
        super().__init__()
        width, eps = config.hidden_size, config.norm_eps
        self.eps, self.mult, self.both = eps, config.residual_mult, config.norms == "both"
        self.mix = MIXERS[layer["type"]](layer["mixer"], width, eps, dtype)
        self.mlp = FEED_FORWARDS[layer["mlp"]["kind"]](layer["mlp"], width, dtype) if layer.get("mlp") is not None else None
        # norm1, norm2: in front of mixer and feed-forward with norms on both sides, else behind them; norm1b, norm2b: behind
        self.norm_names = [n + b for n in (["norm1"] if self.mlp is None else ["norm1", "norm2"]) for b in (["", "b"] if self.both else [""])]
        for name in ("norm1", "norm1b", "norm2", "norm2b"):
            setattr(self, name, _param(width, dtype=torch.float32) if name in self.norm_names else None)

    @property
    def entry_norm(self) -> Optional[torch.Tensor]:
        """The norm between the stream and the mixer."""
        return self.norm1 if self.both else None

    def tensors(self) -> Dict[str, torch.Tensor]:
        out = {name: getattr(self, name) for name in self.norm_names}
        out.update({f"mix.{k}": v for k, v in self.mix.tensors().items()})
        if self.mlp is not None:
            out.update({f"mlp.{k}": v for k, v in self.mlp.tensors().items()})
        return out

    def forward(self, x, xh, state, batch, next_norm: Optional[torch.Tensor] = None):
        """Advances the stream x (fp32) in place.  xh, in the matrices' dtype, is what the mixer reads and, afterwards, what the
        next layer's mixer reads: a copy of the stream (None in fp32, where the stream itself is read), or with norms on both
        sides its norm, for the next layer with weight ``next_norm`` (None: nobody reads it)."""
        src = x if xh is None else xh
        y = self.mix(x, src, state, batch)
        if self.mlp is None:
            self._add(x, xh, y, self.norm1b if self.both else self.norm1, next_norm)
            return
        self._add(x, xh, y, self.norm1b if self.both else self.norm1, self.norm2 if self.both else None)
        y, weights = self.mlp(x, src)
        self._add(x, xh, y, self.norm2b if self.both else self.norm2, next_norm, weights)

    def _add(self, x, xh, y, norm, next_norm, weights=None):
        ops.residual_norm(x, None if self.both and next_norm is None else xh, y, norm, self.eps, weights, self.mult, next_norm)


class HybridModel(nn.Module):
    def __init__(self, config: HybridConfig, dtype: torch.dtype):
        super().__init__()
        self.config, self.dtype = config, dtype
        self.embed = _param(config.vocab_size, config.hidden_size, dtype=dtype)
        self.layers = nn.ModuleList([HybridLayer(l, config, dtype) for l in config.layers])
        self.runs = config.layer_runs()
        self.norm = _param(config.hidden_size, dtype=torch.float32)

    def new_cache(self, num_slots: int = 0) -> HybridCache:
        return HybridCache([self.layers[run.index].mix.spec for run in self.runs], self.dtype, self.embed.device, num_slots)

    def forward(self, ids: torch.Tensor, cache: HybridCache, batch: ops.PackedBatch, layers_out: Optional[List[torch.Tensor]] = None):
        """The fp32 residual stream [T, width padded] behind the last layer; ``layers_out`` receives a copy behind every layer run."""
        cfg, stream = self.config, None
        for n, (run, state) in enumerate(zip(self.runs, cache.layers_state)):
            layer = self.layers[run.index]
            if n == 0 or run.again:
                stream = ops.embed_scaled(ids, self.embed, cfg.embedding_scale, ops.padded(cfg.hidden_size), layer.entry_norm, cfg.norm_eps, add_to=stream)
            following = self.runs[n + 1] if n + 1 < len(self.runs) else None
            layer(*stream, state, batch, self.layers[following.index].entry_norm if following and not following.again else None)
            if layers_out is not None:
                layers_out.append(stream[0][:, :cfg.hidden_size].clone())
        cache.advance(batch)
        return stream[0]


class HybridForCausalLM(GreedyGeneration, nn.Module):
    """Model, head and step function.  ``config_cls`` reads config.json; checkpoint names come from ``tensors``."""
    config_cls = None

    def __init__(self, config: HybridConfig, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{type(self).__name__} runs in bfloat16 or float32, not {dtype}")
        self.config = config
        self.model = HybridModel(config, dtype)
        self.head = None if config.tied_head else _param(config.vocab_size, config.hidden_size, dtype=dtype)

    @staticmethod
    def libraries(config: HybridConfig) -> Tuple[str, ...]:
        """Names (``build.LIBRARIES``) of what a model of this configuration runs on."""
        used = {MIXERS[l["type"]].library for l in config.layers} | {FEED_FORWARDS[l["mlp"]["kind"]].library for l in config.layers if l.get("mlp") is not None}
        return ("hybrid", *sorted(n for n in used if n))

    @property
    def device(self) -> torch.device:
        return self.model.embed.device

    def new_cache(self, num_slots: int = 0) -> HybridCache:
        return self.model.new_cache(num_slots)

    # ---- weights ----------------------------------------------------------------------------------
    def tensors(self) -> Dict[str, torch.Tensor]:
        """Checkpoint name -> the (part of a) parameter it fills (has ``shape`` and ``copy_``)."""
        out = {"embed": self.model.embed, "final.norm": self.model.norm}
        if self.head is not None:
            out["head"] = self.head
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
        logits = F.linear(h, self.model.embed if self.head is None else self.head)
        logits = logits.float() if self.config.logit_softcap is None else ops.soft_cap(logits, self.config.logit_softcap)
        return SimpleNamespace(logits=logits.view(*shape, logits.shape[-1]), past_key_values=cache)
