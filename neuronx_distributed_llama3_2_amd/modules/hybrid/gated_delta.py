"""Mixer "gated delta rule": one projection GEMM, the recurrence over the cached state, one output GEMM."""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn as nn

from ... import ops
from ...ops.delta_rule import DeltaSizes
from .context import StepContext, linear, padded_rows, small


class GatedDeltaMixer(nn.Module):
    in_epilogue = "store"
    recurrent = True   # a step changes what the cache holds of earlier tokens

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, conv: int, eps: float,
                 dtype=torch.bfloat16, device=None):
        super().__init__()
        self.sizes = DeltaSizes(heads, kv_heads, dim, vdim)
        self.taps, self.eps = conv, eps
        # rows: q | k | v | output gate | write strength | decay
        self.in_proj = nn.Linear(width, padded_rows(self.sizes.columns), bias=False, dtype=dtype, device=device)
        self.conv = small(conv, self.sizes.channels, device=device)
        self.a_log = small(heads, device=device)
        self.dt_bias = small(heads, device=device)
        self.out_norm = small(vdim, device=device)
        self.o_proj = nn.Linear(heads * vdim, width, bias=False, dtype=dtype, device=device)
        self.o_bias: Optional[torch.Tensor] = None

    @torch.no_grad()
    def reset_parameters(self) -> None:
        self.conv.uniform_(-0.5, 0.5)
        self.a_log.uniform_(-2.0, 1.0)
        self.dt_bias.uniform_(-3.0, 0.0)
        self.out_norm.fill_(1.0)

    def cache_tensors(self, slots: int, max_len: int, dtype: torch.dtype, device) -> Dict[str, torch.Tensor]:
        s = self.sizes
        return {"state": torch.zeros((slots, s.heads, s.vdim, s.padded_dim), dtype=torch.float32, device=device),
                "ring": torch.zeros((slots, self.taps, s.channels), dtype=dtype, device=device)}

    def max_new_tokens(self, cache: Dict[str, torch.Tensor], max_len: int) -> int:
        return max_len

    @property
    def in_linear(self) -> nn.Linear:
        return self.in_proj

    @property
    def out_linear(self) -> nn.Linear:
        return self.o_proj

    def core(self, proj: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext) -> torch.Tensor:
        """From the input projection's output to the output projection's input."""
        return ops.delta_rule(proj, ctx.B, ctx.T, self.sizes, self.conv, self.a_log, self.dt_bias, self.out_norm,
                              self.eps, ctx.positions, ctx.lengths, ctx.slots, cache["state"], cache["ring"], ctx.fused)

    def forward(self, h: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext) -> torch.Tensor:
        return linear(self.core(linear(h, self.in_proj), cache, ctx), self.o_proj)
