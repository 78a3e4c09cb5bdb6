"""Two mixer cores side by side on the same input: one input projection whose rows are both parts', one
output projection whose columns are both parts'; the scale of each part's output is applied before the
output projection, in the kernels that write its input."""

from __future__ import annotations

from typing import Dict

import torch
import torch.nn as nn

from .context import StepContext, linear, padded_rows


class ParallelMixer(nn.Module):
    def __init__(self, width: int, left: nn.Module, right: nn.Module, left_scale: float, right_scale: float,
                 dtype=torch.bfloat16, device=None):
        super().__init__()
        self.left, self.right = left, right
        self.scales = (left_scale, right_scale)
        self.in_split = padded_rows(left.columns)
        self.out_split = padded_rows(left.outputs)
        self.in_proj = nn.Linear(width, self.in_split + padded_rows(right.columns), bias=False, dtype=dtype, device=device)
        self.o_proj = nn.Linear(self.out_split + padded_rows(right.outputs), width, bias=False, dtype=dtype, device=device)

    @property
    def recurrent(self) -> bool:
        return self.left.recurrent or self.right.recurrent

    @torch.no_grad()
    def reset_parameters(self) -> None:
        self.left.reset_parameters()
        self.right.reset_parameters()

    def cache_tensors(self, slots: int, max_len: int, dtype: torch.dtype, device) -> Dict[str, torch.Tensor]:
        a, b = (m.cache_tensors(slots, max_len, dtype, device) for m in (self.left, self.right))
        assert not set(a) & set(b), "the parts' cache tensors need different names"
        return {**a, **b}

    def max_new_tokens(self, cache: Dict[str, torch.Tensor], max_len: int) -> int:
        return min(m.max_new_tokens(cache, max_len) for m in (self.left, self.right))

    def core(self, buf: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext) -> torch.Tensor:
        """From the input projection's output (which the parts may overwrite) to the output projection's
        input."""
        out = torch.empty((buf.shape[0], self.o_proj.weight.shape[1]), dtype=buf.dtype, device=buf.device)
        for m, lo, hi, src, scale in ((self.left, 0, self.out_split, buf[:, :self.in_split], self.scales[0]),
                                      (self.right, self.out_split, out.shape[1], buf[:, self.in_split:], self.scales[1])):
            if lo + m.outputs < hi:   # padding columns of the projection: their weights are zero
                out[:, lo + m.outputs:hi].zero_()
            m.core(src, cache, ctx, out[:, lo:lo + m.outputs], scale)
        return out

    def forward(self, h: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext) -> torch.Tensor:
        return linear(self.core(linear(h, self.in_proj, ctx.fused), cache, ctx), self.o_proj, ctx.fused)
