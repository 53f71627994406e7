"""Greedy decoding shared by every model family: prompt (whole or in portions), then one token per sequence and step, eagerly
or replayed from a HIP graph."""
from __future__ import annotations

from typing import Optional, Sequence

import torch


class GreedyGeneration:
    """Mixin for a causal LM whose ``forward(input_ids, past_key_values=..., logits_to_keep=...)`` returns ``logits`` and
    ``past_key_values``.  A family whose forward also takes ``lengths`` and ``slots`` serves batches of unequal prompts."""

    def generate(self, input_ids: torch.Tensor, max_new_tokens: int, past_key_values=None, prefill_chunk: int = 0,
                 use_graph: bool = False, lengths: Optional[Sequence[int]] = None):
        """Greedy decoding.  ``prefill_chunk`` > 0 streams the prompt in chunks of that many tokens (with an evicting cache:
        evicting after each, the long-prompt mode of the reference's examples); returns prompt + new tokens.  ``use_graph``:
        the decode steps are captured in a HIP graph once and replayed (``trimkv_amd.graphed.GraphedDecoder``); the cache
        goes back to host-sized launches when the call returns.  ``lengths``: the prompts' lengths when they differ
        (``input_ids`` padded on the right); a list of one tensor per sequence comes back then."""
        with torch.no_grad():
            chunk = prefill_chunk or input_ids.shape[1]
            if lengths is None:
                out = None
                for s in range(0, input_ids.shape[1], chunk):
                    out = self(input_ids[:, s:s + chunk], past_key_values=past_key_values, logits_to_keep=1)
                    past_key_values = out.past_key_values
                last = out.logits[:, -1]
            else:
                last, past_key_values = self._prefill_unequal(input_ids, [int(n) for n in lengths], past_key_values, chunk)
            step, graphed = self, None
            if use_graph and max_new_tokens > 1:
                from .graphed import GraphedDecoder
                graphed = GraphedDecoder(self, past_key_values, logits_to_keep=1)
                step = lambda ids, **_: graphed(input_ids=ids)
            new = []
            try:
                for i in range(max_new_tokens):
                    nxt = last.argmax(-1, keepdim=True)
                    new.append(nxt)
                    if i + 1 < max_new_tokens:
                        last = step(nxt, past_key_values=past_key_values, logits_to_keep=1).logits[:, -1]
            finally:
                if graphed is not None:
                    graphed.close()
            if lengths is None:
                return torch.cat([input_ids] + new, dim=1)
            tail = torch.cat(new, dim=1) if new else input_ids[:, :0]
            return [torch.cat([input_ids[b, :n], tail[b]]) for b, n in enumerate(lengths)]

    def _prefill_unequal(self, input_ids, lengths, cache, chunk):
        """Prompts of different lengths, portion by portion: a step holds the sequences that still have tokens, and each
        leaves its last logits when its prompt ends."""
        if not hasattr(self, "new_cache"):
            raise ValueError(f"{type(self).__name__} keeps one length for all sequences of a batch: prompts must be equally long")
        cache = self.new_cache(len(lengths)) if cache is None else cache
        slots = cache.active if cache.active else cache.allocate(len(lengths))
        slots = list(slots)
        last = [None] * len(lengths)
        for s in range(0, max(lengths), chunk):
            rows = [b for b, n in enumerate(lengths) if n > s]
            part = [min(chunk, lengths[b] - s) for b in rows]
            packed = torch.cat([input_ids[b, s:s + n] for b, n in zip(rows, part)])
            out = self(packed, past_key_values=cache, lengths=part, slots=[slots[b] for b in rows], logits_to_keep=1)
            for i, b in enumerate(rows):
                if s + part[i] == lengths[b]:
                    last[b] = out.logits[i, -1]
        return torch.stack(last), cache
