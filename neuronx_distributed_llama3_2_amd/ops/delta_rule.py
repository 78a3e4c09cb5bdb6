"""Gated delta rule over a cached matrix state (csrc/hybrid/delta_rule.hip): causal depthwise
convolution + silu on q / k / v, unit q / k, the recurrence S <- g S; u = beta (v - S^T k);
S <- S + k u^T; o = S^T q, and the gated head norm.

State of a sequence (its cache slot): `state` [slots, H, V, DP] fp32 (DP = D rounded up to 32) and
`ring` [slots, taps, C], the convolution's inputs by position (p in entry p % taps)."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F

from ._ext import hybrid_ext, use_native


# new tokens per sequence from which the recurrence runs 64 tokens at a time on the matrix cores
# (csrc/hybrid/delta_chunk.hip) instead of token by token
CHUNK_FROM = 32


@dataclass(frozen=True)
class DeltaSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int

    @property
    def channels(self) -> int:   # columns that pass the convolution: q, k, v
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def columns(self) -> int:    # + output gate, write strength, decay
        return self.channels + self.heads * self.vdim + 2 * self.heads

    @property
    def padded_dim(self) -> int:
        return (self.dim + 31) // 32 * 32


def delta_rule(proj: torch.Tensor, B: int, T: int, sizes: DeltaSizes, conv: torch.Tensor, a_log: torch.Tensor,
               dt_bias: torch.Tensor, norm_w: torch.Tensor, eps: float, positions: torch.Tensor,
               lengths: Optional[torch.Tensor], slots: Optional[torch.Tensor], state: torch.Tensor,
               ring: torch.Tensor, fused: bool = True, chunk_from: int = CHUNK_FROM) -> torch.Tensor:
    """proj [B T, >= columns]: [q | k | v | gate | beta | decay] of T new tokens per sequence, the first
    at positions[b] (int64 [B] or [B, T]); lengths [B] int32: valid new tokens (None: T).  conv
    [taps, C] fp32.  Updates state / ring of slots[b]; returns [B T, H V] (padding rows are zero).
    fused: one launch when T == 1.  chunk_from: steps of at least so many tokens take the chunked form."""
    H, G, D, V = sizes.heads, sizes.kv_heads, sizes.dim, sizes.vdim
    y = torch.empty((B * T, H * V), dtype=proj.dtype, device=proj.device)
    if use_native(proj):
        hybrid_ext().delta_rule(proj, B, T, [H, G, D, V], conv, a_log, dt_bias, norm_w, float(eps), positions,
                                lengths, slots, state, ring, y, fused, chunk_from)
        return y
    C, taps = sizes.channels, conv.shape[0]
    y.zero_()
    rep = H // G
    for b in range(B):
        slot = int(slots[b]) if slots is not None else b
        p0 = int(positions.reshape(B, -1)[b, 0])
        n = min(T, int(lengths[b])) if lengths is not None else T
        if n == 0:
            continue
        rows = proj[b * T:b * T + n].float()
        past = torch.zeros((taps - 1, C), dtype=torch.float32)
        for j in range(taps - 1):   # token p0 - (taps - 1 - j)
            p = p0 - (taps - 1 - j)
            if p >= 0:
                past[j] = ring[slot, p % taps].float()
        x = torch.cat([past, rows[:, :C]])
        c = F.silu(sum(x[j:j + n] * conv[j] for j in range(taps)))
        q, k, v = c[:, :G * D].view(n, G, D), c[:, G * D:2 * G * D].view(n, G, D), c[:, 2 * G * D:].view(n, H, V)
        q = (q / torch.sqrt(q.square().sum(-1, keepdim=True) + 1e-6) * D ** -0.5).repeat_interleave(rep, 1)
        k = (k / torch.sqrt(k.square().sum(-1, keepdim=True) + 1e-6)).repeat_interleave(rep, 1)
        beta = torch.sigmoid(rows[:, C + H * V:C + H * V + H])
        g = torch.exp(-torch.exp(a_log) * F.softplus(rows[:, C + H * V + H:C + H * V + 2 * H] + dt_bias))
        S = state[slot, :, :, :D].clone() if p0 > 0 else torch.zeros((H, V, D))
        o = torch.empty((n, H, V))
        for t in range(n):
            S = S * g[t, :, None, None]
            u = beta[t, :, None] * (v[t] - torch.matmul(S, k[t].unsqueeze(-1)).squeeze(-1))
            S = S + u.unsqueeze(-1) * k[t].unsqueeze(1)
            o[t] = torch.matmul(S, q[t].unsqueeze(-1)).squeeze(-1)
        state[slot, :, :, :D] = S
        for t in range(max(0, n - taps), n):
            ring[slot, (p0 + t) % taps] = proj[b * T + t, :C]
        o = o / torch.sqrt(o.square().mean(-1, keepdim=True) + eps) * norm_w
        y[b * T:b * T + n] = (o * F.silu(rows[:, C:C + H * V]).view(n, H, V)).reshape(n, H * V).to(y.dtype)
    return y
