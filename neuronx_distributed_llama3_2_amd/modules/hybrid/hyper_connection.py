"""Weights of one hyper-connection: how a sublayer reads the residual streams and how its output and
the old streams make the new ones (ops.hyper_step does the arithmetic)."""

from __future__ import annotations

import torch
import torch.nn as nn

from .context import small


class HyperConnection(nn.Module):
    def __init__(self, streams: int, device=None):
        super().__init__()
        self.read = small(streams, device=device)
        self.mix = small(streams, streams, device=device)    # [from, to]
        self.write = small(streams, device=device)

    @torch.no_grad()
    def reset_parameters(self) -> None:
        """An ordinary residual in every stream."""
        self.read.fill_(1.0 / self.read.numel())
        self.write.fill_(1.0)
        self.mix.zero_().fill_diagonal_(1.0)
