"""Mixer core "window and pooled blocks": grouped-query attention over a sliding window and the means of
the blocks before it; norms over whole projections, values = keys as projected, no positions."""

from __future__ import annotations

from typing import Dict

import torch
import torch.nn as nn

from ... import ops
from ...ops.pooled_attention import PooledRule, PooledSizes
from .context import StepContext, small
from .differential_attention import RING_SLACK


class PooledAttention(nn.Module):
    """Between the projections of a mixer: `core` reads `columns` of the input projection's output and
    writes `outputs` columns of the output projection's input."""

    recurrent = False

    def __init__(self, heads: int, kv_heads: int, dim: int, scale: float, window: int, pool: int, eps: float, device=None):
        super().__init__()
        self.sizes = PooledSizes(heads, kv_heads, dim)
        self.rule = PooledRule(scale, window, pool, eps)
        self.q_norm = small(heads * dim, device=device)
        self.k_norm = small(kv_heads * dim, device=device)

    @property
    def columns(self) -> int:
        return self.sizes.columns

    @property
    def outputs(self) -> int:
        return self.sizes.q_columns

    @torch.no_grad()
    def reset_parameters(self) -> None:
        self.q_norm.fill_(1.0)
        self.k_norm.fill_(1.0)

    def cache_tensors(self, slots: int, max_len: int, dtype: torch.dtype, device) -> Dict[str, torch.Tensor]:
        s, r = self.sizes, self.rule
        cap = min(max_len, (max(r.window, r.pool) + RING_SLACK + 63) // 64 * 64)
        z = lambda n: torch.zeros((slots, s.kv_heads, n, s.dim), dtype=dtype, device=device)  # noqa: E731
        blocks = max(1, max_len // r.pool)
        return {"k": z(cap), "v": z(cap), "pk": z(blocks), "pv": z(blocks),
                "tickets": torch.zeros(slots * s.heads, dtype=torch.int32, device=device)}

    def max_new_tokens(self, cache: Dict[str, torch.Tensor], max_len: int) -> int:
        """Tokens one decode step may bring: the ring must still hold what the first of them sees, and every
        token of the blocks that they complete."""
        cap = cache["k"].shape[2]
        return max_len if cap >= max_len else cap - max(self.rule.window, self.rule.pool) + 1

    def core(self, buf: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext, out: torch.Tensor,
             out_scale: float = 1.0) -> None:
        if ctx.fused and ctx.T == 1 and not ctx.prompt and ctx.lengths is None:
            ops.pooled_decode(buf, self.sizes, self.rule, self.q_norm, self.k_norm, ctx.positions, ctx.slots, cache, out, out_scale)
            return
        kn = ops.pooled_prep_(buf, ctx.B, ctx.T, self.sizes, self.rule, self.q_norm, self.k_norm, ctx.positions, ctx.lengths,
                              ctx.slots, cache, ctx.prompt)
        ops.pooled_attention(buf, kn, ctx.B, ctx.T, self.sizes, self.rule, ctx.positions, ctx.lengths, ctx.slots, cache,
                             ctx.prompt, out, out_scale, ctx.fused)
