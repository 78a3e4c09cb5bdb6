"""Feed-forward of routed experts with a sigmoid router over groups of experts, clamped gated
activations and an optional shared expert with a gate of its own."""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn as nn

from ... import ops
from ...ops.experts import FEW_ROWS, RouterRule
from ...ops.gemm import linear_f32
from .context import linear, padded_rows


class RoutedExperts(nn.Module):
    def __init__(self, width: int, rule: RouterRule, ff: int, limit: float, shared_ff: int = 0, shared_limit: float = 0.0,
                 dtype=torch.bfloat16, device=None):
        super().__init__()
        self.rule, self.limit, self.shared_ff, self.shared_limit = rule, limit, shared_ff, shared_limit
        E = rule.experts
        new = lambda *s: nn.Parameter(torch.empty(s, dtype=dtype, device=device), requires_grad=False)  # noqa: E731
        # rows: one per expert, then the shared expert's gate
        self.router = nn.Linear(width, padded_rows(E + (1 if shared_ff else 0)), bias=False, dtype=dtype, device=device)
        self.gate_up = new(E, 2 * ff, width)
        self.down = new(E, width, ff)
        self.shared_up: Optional[nn.Linear] = None
        if shared_ff:
            self.shared_up = nn.Linear(width, 2 * shared_ff, bias=False, dtype=dtype, device=device)
            self.shared_down = nn.Linear(shared_ff, width, bias=False, dtype=dtype, device=device)

    @torch.no_grad()
    def reset_parameters(self) -> None:
        self.gate_up.normal_(0.0, self.gate_up.shape[2] ** -0.5)
        self.down.normal_(0.0, self.down.shape[2] ** -0.5)

    def forward(self, h: torch.Tensor, fused: bool = True) -> Dict[str, object]:
        """What ops.residual_norms adds to the residual: the outputs of (token, choice) pairs, weighted,
        where each is, and the shared expert's output.  fused: a few tokens take the unsorted kernels."""
        shared = (self.shared_up.weight, self.shared_down.weight) if self.shared_up is not None else (None, None)
        if fused and ops.experts_few_supported(h, self.gate_up, self.down, *shared):
            inside = h.shape[0] <= FEW_ROWS
            gate = torch.empty(h.shape[0], dtype=torch.float32, device=h.device) if shared[0] is not None and not inside else None
            pairs = ops.experts_few(h, self.router.weight, self.rule, self.gate_up, self.down, self.limit,
                                    *(shared if inside else (None, None)), self.shared_limit, gate)
            return dict(pairs=pairs, adds=[] if gate is None else [self._shared(h, gate, False)])
        logits = linear_f32(h, self.router.weight)
        r = ops.route(logits, self.rule)
        a = ops.clamped_glu(ops.expert_linear_rows(h, self.gate_up, r.offs, r.token), self.limit, r.weight)
        out: Dict[str, object] = dict(pairs=ops.expert_linear_rows(a, self.down, r.offs), inverse=r.inverse, adds=[])
        if self.shared_up is not None:
            out["adds"] = [self._shared(h, logits[:, self.rule.experts], True)]
        return out

    def _shared(self, h: torch.Tensor, gate: torch.Tensor, sigmoid: bool) -> torch.Tensor:
        return linear(ops.clamped_glu(linear(h, self.shared_up), self.shared_limit, gate, sigmoid=sigmoid), self.shared_down)
