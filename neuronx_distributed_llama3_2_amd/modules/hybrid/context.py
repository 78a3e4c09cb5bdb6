"""What a mixer needs to know about the step it runs in."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch


@dataclass
class StepContext:
    """T new tokens for each of B sequences (row b * T + t of every activation).  positions: int64, the
    first new token's in column 0; lengths [B] int32: valid new tokens (None: all T); slots [B] int32
    cache slots (None: 0..B-1); prompt: every sequence starts at position 0 in this step."""

    B: int
    T: int
    positions: torch.Tensor
    lengths: Optional[torch.Tensor]
    slots: Optional[torch.Tensor]
    prompt: bool
    fused: bool = True


# rows of a fused projection are padded to this, so that every row of its output is 16-byte aligned
ROW_ALIGN = 16


def padded_rows(n: int) -> int:
    return (n + ROW_ALIGN - 1) // ROW_ALIGN * ROW_ALIGN


# rows up to which a projection is a dot product a wave (csrc/hybrid/gemv_hyper.hip), and up to which it is
# 16 weight rows a workgroup (csrc/hybrid/expert_decode.hip)
FEW_ROWS, SOME_ROWS = 2, 16


def few_rows(x: torch.Tensor, w: torch.Tensor, limit: int = FEW_ROWS) -> bool:
    return x.is_cuda and x.shape[0] <= limit and x.dtype == w.dtype == torch.bfloat16 and w.shape[1] % 8 == 0 and x.is_contiguous()


def linear(x: torch.Tensor, mod: torch.nn.Module, fused: bool = False) -> torch.Tensor:
    """x [M, K] @ mod.weight^T: through the module's packed copy when the layout pass chose it; fused: a few
    rows by the kernels that stream the weights."""
    from ... import ops
    from ...trace.weight_layout import packed_linear

    if fused and few_rows(x, mod.weight, SOME_ROWS):
        return ops.decode_linear(mod.weight, x) if x.shape[0] <= FEW_ROWS else ops.linear_few(x, mod.weight)
    return packed_linear(mod, x, mod.weight)


def small(*shape, device=None) -> torch.nn.Parameter:
    """A small parameter that enters 32-bit computations: kept in fp32 whatever the model's dtype."""
    return torch.nn.Parameter(torch.empty(*shape, dtype=torch.float32, device=device), requires_grad=False)
