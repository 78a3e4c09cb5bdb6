"""Per-layer cache of a decoder whose layers keep different things of a sequence: keys and values of
every token (attention), of the last window of tokens (windowed attention), or a fixed-size state
(recurrent mixers).  Each mixer names its tensors (`cache_tensors`); all have the cache slot as their
first dimension, so a slot is one sequence's place in every layer.

Nothing has to be cleared when a slot is given to another sequence: positions tell the kernels what
belongs to the sequence, and a recurrent mixer starts from zero at position 0."""

from __future__ import annotations

from typing import Dict, List

import torch


class LayerCache:
    def __init__(self, mixers, slots: int, max_len: int, dtype: torch.dtype, device):
        self.slots, self.max_len, self.dtype, self.device = slots, max_len, dtype, torch.device(device)
        self.layers: List[Dict[str, torch.Tensor]] = [m.cache_tensors(slots, max_len, dtype, device) for m in mixers]
        # most new tokens one decode step may bring (forward_tokens cuts longer ones)
        self.max_step = min([m.max_new_tokens(c, max_len) for m, c in zip(mixers, self.layers)], default=max_len)
        # layers whose cache a step overwrites: a full-length key cache only gains entries
        self._overwritten = [i for i, (m, c) in enumerate(zip(mixers, self.layers))
                             if m.recurrent or any(c[n].shape[2] < max_len for n in ("k", "v") if n in c)]

    def matches(self, slots: int, max_len: int, dtype: torch.dtype, device) -> bool:
        return (self.slots, self.max_len, self.dtype, self.device) == (slots, max_len, dtype, torch.device(device))

    def __getitem__(self, i: int) -> Dict[str, torch.Tensor]:
        return self.layers[i]

    def zero_(self) -> None:
        for c in self.layers:
            for t in c.values():
                t.zero_()

    def save(self) -> list:
        """Copy of everything that running a step again would not simply write again."""
        return [(i, {n: t.clone() for n, t in self.layers[i].items()}) for i in self._overwritten]

    def load(self, saved: list) -> None:
        for i, c in saved:
            for n, t in c.items():
                self.layers[i][n].copy_(t)

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for c in self.layers for t in c.values())
