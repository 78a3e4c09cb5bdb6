"""Feed-forward with the squared ReLU: down(relu(up x)^2)."""

from __future__ import annotations

import torch
import torch.nn as nn

from ... import ops
from .context import linear


class SquaredReluMLP(nn.Module):
    in_epilogue = "relu2"   # of the fused decode projection (ops.decode_linear)
    o_bias = None

    def __init__(self, width: int, ff: int, dtype=torch.bfloat16, device=None):
        super().__init__()
        self.up_proj = nn.Linear(width, ff, bias=False, dtype=dtype, device=device)
        self.down_proj = nn.Linear(ff, width, bias=False, dtype=dtype, device=device)

    @property
    def in_linear(self) -> nn.Linear:
        return self.up_proj

    @property
    def out_linear(self) -> nn.Linear:
        return self.down_proj

    def core(self, a: torch.Tensor, cache, ctx) -> torch.Tensor:
        return a

    def forward(self, h: torch.Tensor, cache=None, ctx=None) -> torch.Tensor:
        return linear(ops.relu_squared(linear(h, self.up_proj)), self.down_proj)
