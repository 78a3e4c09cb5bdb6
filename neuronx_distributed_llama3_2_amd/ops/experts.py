"""Routed experts of inference decoders (csrc/hybrid/moe_route.hip, expert_decode.hip and the grouped GEMMs):
sigmoid router with groups of experts, clamped gated activation, all on the device without a host sync."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from ._ext import hybrid_ext, use_native


@dataclass(frozen=True)
class RouterRule:
    """The `top` experts of largest sigmoid score among the experts of the `keep` best of `groups` groups
    (by the sum of a group's two largest scores); weights: their scores over the scores' sum, times scale."""

    experts: int
    top: int
    scale: float = 1.0
    groups: int = 1
    keep: int = 1

    def as_list(self):
        return [self.experts, self.top, self.groups, self.keep]


@dataclass
class Routing:
    """(token, choice) pairs sorted by expert: expert e has rows offs[e] .. offs[e + 1]; row r belongs to
    token[r] and has weight[r]; choice j of token m is row inverse[m, j].  All int32 / fp32."""

    token: torch.Tensor
    weight: torch.Tensor
    inverse: torch.Tensor
    offs: torch.Tensor


def route(logits: torch.Tensor, rule: RouterRule) -> Routing:
    """logits [M, >= experts] fp32."""
    M, P = logits.shape[0], logits.shape[0] * rule.top
    if use_native(logits):
        new = lambda n, dt: torch.empty(n, dtype=dt, device=logits.device)  # noqa: E731
        r = Routing(new(P, torch.int32), new(P, torch.float32), new((M, rule.top), torch.int32),
                    new(rule.experts + 1, torch.int32))
        hybrid_ext().moe_route(logits, rule.as_list(), rule.scale, r.token, r.weight, r.inverse, r.offs)
        return r
    s = torch.sigmoid(logits[:, :rule.experts].float())
    per = rule.experts // rule.groups
    best2 = s.view(M, rule.groups, per).topk(min(2, per), -1).values.sum(-1)
    kept = torch.zeros((M, rule.groups), dtype=torch.bool).scatter_(1, best2.topk(rule.keep, -1).indices, True)
    w, index = s.masked_fill(~kept.repeat_interleave(per, 1), -1.0).topk(rule.top, -1)
    w = w / (w.sum(-1, keepdim=True) + 1e-20) * rule.scale
    flat = index.reshape(-1)
    order = torch.argsort(flat, stable=True)
    inverse = torch.empty_like(order)
    inverse[order] = torch.arange(P)
    offs = torch.zeros(rule.experts + 1, dtype=torch.int32)
    offs[1:] = torch.cumsum(torch.bincount(flat, minlength=rule.experts), 0)
    return Routing((order // rule.top).int(), w.reshape(-1)[order], inverse.view(M, rule.top).int(), offs)


def clamped_glu(gu: torch.Tensor, limit: float, weight: Optional[torch.Tensor] = None, sigmoid: bool = False) -> torch.Tensor:
    """gu [R, 2 F] = [gate | up] -> g sigmoid(1.702 g) (u + 1) with g = min(gate, limit), u = up clamped to
    +-limit; times weight[r] (fp32 [R], any stride), or its sigmoid."""
    R, F = gu.shape[0], gu.shape[1] // 2
    if use_native(gu):
        y = torch.empty((R, F), dtype=gu.dtype, device=gu.device)
        hybrid_ext().clamped_glu(gu, float(limit), weight, sigmoid, y)
        return y
    g, u = gu[:, :F].float().clamp(max=limit), gu[:, F:].float().clamp(-limit, limit)
    y = g * torch.sigmoid(1.702 * g) * (u + 1)
    if weight is not None:
        y = y * (torch.sigmoid(weight) if sigmoid else weight).unsqueeze(1)
    return y.to(gu.dtype)


def expert_linear_rows(x: torch.Tensor, w: torch.Tensor, offs: torch.Tensor, token: Optional[torch.Tensor] = None) -> torch.Tensor:
    """y[r] = x[token[r]] (or x[r]) w[e]^T for the rows r of expert e; w [E, N, K].  bf16 with K and N
    multiples of 8: the grouped matrix-core GEMM over gathered rows; else a kernel for any size and type."""
    E, N, K = w.shape
    P = x.shape[0] if token is None else token.numel()
    if use_native(x, w):
        H = hybrid_ext()
        y = torch.empty((P, N), dtype=x.dtype, device=x.device)
        if x.dtype == torch.bfloat16 and K % 8 == 0 and N % 8 == 0:
            if token is not None:
                xs = torch.empty((P, K), dtype=x.dtype, device=x.device)
                H.gather_rows(x, token, xs)
                x = xs
            H.grouped_linear(x, w, offs, y)
        else:
            H.expert_rows(x, w, offs, token, y)
        return y
    xs = x if token is None else x[token.long()]
    y = torch.empty((P, N), dtype=x.dtype)
    b = offs.tolist()
    for e in range(E):
        y[b[e]:b[e + 1]] = torch.nn.functional.linear(xs[b[e]:b[e + 1]], w[e])
    return y


# tokens up to which the experts run unsorted, and up to which dense weights are streamed beside them
# (csrc/hybrid/expert_decode.hip)
FEW_TOKENS, FEW_ROWS = 64, 16


def linear_few(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x [M, K] w^T for up to FEW_ROWS rows (GPU, bf16, K a multiple of 8): the weights are streamed once."""
    y = torch.empty((x.shape[0], w.shape[0]), dtype=x.dtype, device=x.device)
    hybrid_ext().linear_few(x, w, y)
    return y


def experts_few_supported(h: torch.Tensor, *weights: Optional[torch.Tensor]) -> bool:
    return use_native(h) and h.shape[0] <= FEW_TOKENS and h.dtype == torch.bfloat16 and \
        all(w is None or w.dtype == torch.bfloat16 and w.shape[-1] % 8 == 0 for w in weights)


def experts_few(h: torch.Tensor, router: torch.Tensor, rule: RouterRule, gate_up: torch.Tensor, down: torch.Tensor, limit: float,
                shared_up: Optional[torch.Tensor] = None, shared_down: Optional[torch.Tensor] = None,
                shared_limit: float = 0.0, gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """A whole routed feed-forward for a few tokens (GPU, bf16) in three launches.  router [>= E (+ 1), W]: the
    experts' rows, then the shared expert's gate.  Returns [M (top + 1), W]: for each token its experts'
    weighted outputs and then its shared expert's; their sum is the feed-forward's output.  gate (fp32 [M],
    instead of the shared expert's weights): receives its gate, and the rows are the experts' alone."""
    slots = rule.top + (0 if shared_up is None else 1)
    y = torch.empty((h.shape[0] * slots, h.shape[1]), dtype=h.dtype, device=h.device)
    hybrid_ext().experts_few(h, router, rule.as_list(), rule.scale, gate_up, down, float(limit), shared_up, shared_down,
                             float(shared_limit), gate, y)
    return y
