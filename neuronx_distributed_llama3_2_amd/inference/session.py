"""A batch of requests over an inference application, fed with given tokens: start a batch with whole
prompts, then go on by one token per request, requests leaving as they end.  It drives the
application's own context encoding and token generation, and hands out the cache slots."""

from __future__ import annotations

from typing import Dict, Iterable, List, Optional, Sequence, Tuple

import torch


class BatchSession:
    def __init__(self, app):
        self.app = app
        self._slot: Dict[str, int] = {}
        self._len: Dict[str, int] = {}
        self._free: List[int] = list(range(app.max_batch))

    def _claim(self, n: int) -> List[int]:
        if n > len(self._free):
            if self._slot:
                raise ValueError(f"{n} requests for {len(self._free)} free cache slots")
            self.app.ensure_slots(n)
            self._free = list(range(self.app.max_batch))
        return [self._free.pop(0) for _ in range(n)]

    def step(self, entries: Sequence[Tuple[str, Sequence[int], Sequence[int]]]) -> Optional[torch.Tensor]:
        """entries: (request, its next tokens, places among them whose logits are wanted), either all new
        requests or all running ones with one token each.  Returns the wanted logits [R, V] in that order
        (None if there are none)."""
        if not entries:
            return None
        new = [r not in self._slot for r, _, _ in entries]
        if len({r for r, _, _ in entries}) != len(entries) or any(not t for _, t, _ in entries):
            raise ValueError("a request appears twice in a step, or brings no tokens")
        if all(new):
            if self._slot:
                raise ValueError("requests are still running; a new batch starts when they have ended")
            return self._start(entries)
        if any(new) or any(len(t) != 1 for _, t, _ in entries):
            raise ValueError("a step starts a batch, or brings one token for each of some running requests")
        return self._next(entries)

    def _start(self, entries) -> Optional[torch.Tensor]:
        B, T = len(entries), max(len(t) for _, t, _ in entries)
        limit = self.app.config.max_length
        if T > limit:
            raise ValueError(f"a prompt of {T} tokens exceeds {limit}")
        ids = torch.zeros((B, T), dtype=torch.long)
        mask = torch.zeros((B, T), dtype=torch.long)
        for b, (_, tokens, _) in enumerate(entries):
            ids[b, :len(tokens)] = torch.as_tensor(tokens)
            mask[b, :len(tokens)] = 1
        slots = self._claim(B)
        want = [(b, p) for b, (_, tokens, ps) in enumerate(entries) for p in self._places(tokens, ps)]
        rows = torch.tensor(want or [(0, 0)], dtype=torch.long)   # a forward has at least one logit row
        logits = self.app._context_encode(ids, mask, seq_ids=torch.tensor(slots, dtype=torch.int32), want=rows)
        for slot, (r, tokens, _) in zip(slots, entries):
            self._slot[r], self._len[r] = slot, len(tokens)
        return logits if want else None

    def _next(self, entries) -> Optional[torch.Tensor]:
        for r, _, _ in entries:
            if self._len[r] >= self.app.config.max_length:
                raise ValueError(f"request {r} exceeds {self.app.config.max_length} tokens")
        ids = torch.tensor([[t[0]] for _, t, _ in entries], dtype=torch.long)
        pos = torch.tensor([[self._len[r]] for r, _, _ in entries], dtype=torch.long)
        slots = torch.tensor([self._slot[r] for r, _, _ in entries], dtype=torch.int32)
        logits = self.app._token_generate(ids, position_ids=pos, seq_ids=slots)[:, -1]
        for r, _, _ in entries:
            self._len[r] += 1
        want = [b for b, (_, tokens, ps) in enumerate(entries) for _ in self._places(tokens, ps)]
        return logits[want] if want else None

    @staticmethod
    def _places(tokens, places):
        for p in places:
            if not 0 <= p < len(tokens):
                raise ValueError(f"place {p} is not among {len(tokens)} tokens")
        return places

    def end(self, requests: Iterable[str]) -> None:
        """Give back what these requests hold."""
        for r in requests:
            self._free.append(self._slot.pop(r))
            del self._len[r]
        self._free.sort()
