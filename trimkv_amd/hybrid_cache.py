"""What the sequences of a hybrid decoder leave behind from step to step: window rings of attention layers and fp32 states of
recurrent layers, both of fixed size per sequence however long it gets.

A sequence owns one slot; slot ``i`` of every layer's tensors is its share.  Slots are handed out and taken back on the host
(``allocate``, ``release``); a slot that is used again is not cleared: its token count is set to 0, and no kernel reads the
contents of a slot with no tokens.  Token and step counts live on the device (``seen``) beside exact host mirrors, so a decode
step's launches depend on no host-side length and can be replayed from a HIP graph.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch

from . import _lib
from .hybrid_ops import PackedBatch, advance

try:
    from transformers.cache_utils import Cache as _CacheBase
except Exception:  # pragma: no cover - transformers is optional
    class _CacheBase:  # type: ignore
        pass


class HybridCache(_CacheBase):
    """``specs``: one state specification per layer (``WindowSpec``, ``MlstmSpec``; anything with ``state_shapes``)."""

    def __init__(self, specs: Sequence, dtype: torch.dtype, device="cuda", num_slots: int = 0) -> None:
        self.specs, self.dtype, self.device = tuple(specs), dtype, torch.device(device)
        if self.device.type != "cuda":
            raise _lib.TrimKVLibraryError(f"HybridCache on {self.device}: the hybrid decoders run on the GPU only (no CPU path)")
        self.num_slots = 0
        self.layers_state: List[Dict[str, torch.Tensor]] = [{} for _ in self.specs]
        self.seen = torch.zeros(0, 2, dtype=torch.int32, device=self.device)
        self.tokens_seen: List[int] = []           # host mirror of seen[:, 0]
        self.active: List[int] = []                # slots in use, in batch order
        self._free: List[int] = []
        self._batches: Dict[Tuple, Tuple[torch.Tensor, torch.Tensor]] = {}
        self.lengths_on_device = False
        if num_slots:
            self._grow(num_slots)

    # ---- slots ----------------------------------------------------------------------------------
    def _grow(self, num_slots: int) -> None:
        if self.lengths_on_device:
            raise RuntimeError("HybridCache: slots cannot be added while steps are replayed from a graph")
        old = self.num_slots
        for spec, state in zip(self.specs, self.layers_state):
            for name, (shape, dtype) in spec.state_shapes(num_slots, self.dtype).items():
                new = torch.zeros(shape, dtype=dtype, device=self.device)
                if old:
                    new.narrow(1 if name == "nm" else 0, 0, old).copy_(state[name])
                state[name] = new
        seen = torch.zeros(num_slots, 2, dtype=torch.int32, device=self.device)
        seen[:old] = self.seen
        self.seen = seen
        self.tokens_seen += [0] * (num_slots - old)
        self._free += range(old, num_slots)
        self.num_slots = num_slots
        self._batches.clear()

    def allocate(self, n: int) -> List[int]:
        """``n`` fresh sequences at the end of the batch; returns their slots."""
        if len(self._free) < n:
            self._grow(max(self.num_slots - len(self._free) + n, self.num_slots + self.num_slots // 2))
        slots, self._free = self._free[:n], self._free[n:]
        self.seen[torch.tensor(slots, device=self.device)] = 0
        for s in slots:
            self.tokens_seen[s] = 0
        self.active += slots
        return slots

    def release(self, slots: Sequence[int]) -> None:
        """The sequences in these slots are finished."""
        for s in slots:
            self.active.remove(s)
        self._free += list(slots)

    def batch(self, lengths: Sequence[int], slots: Optional[Sequence[int]] = None) -> PackedBatch:
        """The packed description of a step that brings ``lengths[b]`` tokens to each of ``slots`` (default: all active, in order)."""
        slots = tuple(self.active if slots is None else slots)
        lengths = tuple(int(n) for n in lengths)
        if len(slots) != len(lengths):
            raise ValueError(f"{len(lengths)} sequences for {len(slots)} cache slots")
        if len(set(slots)) != len(slots) or any(s not in self.active for s in slots):
            raise ValueError("cache slots must be distinct and allocated")
        if not lengths or min(lengths) < 1:
            raise ValueError("every sequence of a step needs at least one token")
        hit = self._batches.get((lengths, slots))
        if hit is None:
            if len(self._batches) > 64:
                self._batches.clear()
            cu = [0]
            for n in lengths:
                cu.append(cu[-1] + n)
            both = torch.tensor(cu + list(slots), dtype=torch.int32).to(self.device)
            hit = self._batches[(lengths, slots)] = (both[:len(cu)], both[len(cu):])
        return PackedBatch(lengths, slots, hit[0], hit[1], self.seen, self.num_slots)

    def advance(self, batch: PackedBatch) -> None:
        """The step is done: its tokens count from now on."""
        advance(batch)
        for s, n in zip(batch.slots, batch.lengths):
            self.tokens_seen[s] += n

    # ---- the queries and batch utilities of the other caches -------------------------------------
    def __len__(self) -> int:
        return len(self.specs)

    def get_seq_length(self, layer_idx: Optional[int] = None) -> int:
        """Tokens seen by the longest active sequence."""
        return max((self.tokens_seen[s] for s in self.active), default=0)

    def get_cache_length(self, layer_idx: int = 0) -> int:
        """Rows (attention layer) the longest sequence holds in ``layer_idx``; 0 for a recurrent layer."""
        rows = getattr(self.specs[layer_idx], "rows", 0)
        return min(rows, self.get_seq_length())

    def memory_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for state in self.layers_state for t in state.values())

    def batch_select_indices(self, indices: torch.Tensor) -> None:
        """Only keep ``indices`` along the batch axis; an index that comes again gets a slot of its own with a copy."""
        rows = [self.active[int(i)] for i in indices]
        dropped = [s for s in self.active if s not in rows]
        self.release(dropped)
        order, taken = [], set()
        for s in rows:
            if s not in taken:
                taken.add(s)
                order.append(s)
            else:
                (new,) = self.allocate(1)
                for state in self.layers_state:
                    for name, t in state.items():
                        if name == "nm":
                            t[:, new] = t[:, s]
                        else:
                            t[new] = t[s]
                self.seen[new] = self.seen[s]
                self.tokens_seen[new] = self.tokens_seen[s]
                order.append(new)
        self.active = order

    # ---- decode steps that a HIP graph can replay -------------------------------------------------
    def begin_device_steps(self, *_) -> None:
        """Every decode step already enqueues the same launches with the same arguments; from here on storage must not move."""
        if not self.active or any(self.tokens_seen[s] == 0 for s in self.active):
            raise RuntimeError("begin_device_steps: every sequence must hold a prompt first")
        self.lengths_on_device = True

    def end_device_steps(self) -> None:
        self.lengths_on_device = False

    def mirror_snapshot(self):
        return list(self.tokens_seen)

    def mirror_restore(self, snap) -> None:
        self.tokens_seen = list(snap)

    def advance_decode_mirrors(self, *_) -> None:
        for s in self.active:
            self.tokens_seen[s] += 1
