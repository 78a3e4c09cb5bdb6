"""Mixer core "generalised delta rule": decay and removal per key channel over a cached matrix state."""

from __future__ import annotations

from typing import Dict

import torch
import torch.nn as nn

from ... import ops
from ...ops.channel_delta import ChannelDeltaSizes
from .context import StepContext, small


class ChannelDelta(nn.Module):
    """Between the projections of a mixer (as PooledAttention)."""

    recurrent = True   # a step changes what the cache holds of earlier tokens

    def __init__(self, heads: int, dim: int, rank: int, eps: float, dtype=torch.bfloat16, device=None):
        super().__init__()
        self.sizes, self.eps = ChannelDeltaSizes(heads, dim, rank), eps
        n = heads * dim
        self.w2 = nn.Parameter(torch.empty((n, rank), dtype=dtype, device=device), requires_grad=False)
        self.w0 = small(n, device=device)
        self.a_bias = small(n, device=device)
        self.out_norm = small(n, device=device)

    @property
    def columns(self) -> int:
        return self.sizes.columns

    @property
    def outputs(self) -> int:
        return self.sizes.width

    @torch.no_grad()
    def reset_parameters(self) -> None:
        self.w2.normal_(0.0, self.sizes.rank ** -0.5)
        self.w0.uniform_(-4.0, 0.0)
        self.a_bias.zero_()
        self.out_norm.fill_(1.0)

    def cache_tensors(self, slots: int, max_len: int, dtype: torch.dtype, device) -> Dict[str, torch.Tensor]:
        s = self.sizes
        return {"state": torch.zeros((slots, s.heads, s.dim, s.padded_dim), dtype=torch.float32, device=device)}

    def max_new_tokens(self, cache: Dict[str, torch.Tensor], max_len: int) -> int:
        return max_len

    def core(self, buf: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext, out: torch.Tensor,
             out_scale: float = 1.0) -> None:
        ops.channel_delta(buf, ctx.B, ctx.T, self.sizes, self.w2, self.w0, self.a_bias, self.out_norm, self.eps, ctx.positions,
                          ctx.lengths, ctx.slots, cache["state"], out, out_scale)
