"""Generalised delta rule over a cached matrix state (csrc/hybrid/channel_delta*.hip): decay w and removal
rate a per head and key channel,

  S <- diag(w) S - (a * u) (u^T S) + k v^T  (both terms read the old state);  o = S^T r

with u the unit vector of k, w = exp(-e^(-1/2) sigmoid(W2 tanh(low) + w0)), a = sigmoid(. + bias); then the
gated head norm.  State of a sequence (its cache slot): `state` [slots, H, D, DP] fp32, [value channel,
key channel] with the key channels rounded up to DP = 32 n."""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Optional

import torch

from ._ext import hybrid_ext, use_native

# new tokens per sequence from which the recurrence runs in chunks on the matrix cores
# (csrc/hybrid/channel_delta_chunk.hip) instead of token by token
CHUNK_FROM = 16


@dataclass(frozen=True)
class ChannelDeltaSizes:
    heads: int
    dim: int
    rank: int       # of the decay's projection

    @property
    def width(self) -> int:
        return self.heads * self.dim

    @property
    def columns(self) -> int:    # r | k | v | output gate | removal | low-rank decay
        return 5 * self.width + self.rank

    @property
    def padded_dim(self) -> int:
        return (self.dim + 31) // 32 * 32

    def as_list(self):
        return [self.heads, self.dim, self.rank]


def channel_delta(proj: torch.Tensor, B: int, T: int, sizes: ChannelDeltaSizes, w2: torch.Tensor, w0: torch.Tensor,
                  a_bias: torch.Tensor, norm_w: torch.Tensor, eps: float, positions: torch.Tensor,
                  lengths: Optional[torch.Tensor], slots: Optional[torch.Tensor], state: torch.Tensor, out: torch.Tensor,
                  out_scale: float = 1.0, chunk_from: int = CHUNK_FROM) -> None:
    """proj [B T, >= columns]: [r | k | v | gate | removal | low] of T new tokens per sequence, the first at
    positions[b] (int64 [B] or [B, T]); lengths [B] int32: valid new tokens (None: T).  w2 [H D, rank] in
    the activation type, the other weights fp32 [H D].  Updates the state of slots[b]; out [B T, H D] =
    out_scale * the mixer's output before its projection (padding rows are zero).  chunk_from: steps of at
    least so many tokens take the chunked form."""
    H, D, N = sizes.heads, sizes.dim, sizes.rank
    if use_native(proj):
        hybrid_ext().channel_delta(proj, B, T, sizes.as_list(), w2, w0, a_bias, norm_w, float(eps), positions, lengths, slots,
                                   state, out, float(out_scale), chunk_from)
        return
    out.zero_()
    W = sizes.width
    for b in range(B):
        slot = int(slots[b]) if slots is not None else b
        p0 = int(positions.reshape(B, -1)[b, 0])
        n = min(T, int(lengths[b])) if lengths is not None else T
        if n == 0:
            continue
        x = proj[b * T:b * T + n].float()
        r, k, v, g, a = (x[:, i * W:(i + 1) * W].reshape(n, H, D) for i in range(5))
        low = torch.tanh(x[:, 5 * W:5 * W + N])
        w = torch.exp(-math.exp(-0.5) * torch.sigmoid(low @ w2.float().t() + w0)).view(n, H, D)
        a = torch.sigmoid(a + a_bias.view(H, D))
        u = k / torch.sqrt(k.square().sum(-1, keepdim=True) + 1e-6)
        S = state[slot, :, :, :D].clone() if p0 > 0 else torch.zeros((H, D, D))   # [head, value, key]
        o = torch.empty((n, H, D))
        for t in range(n):
            z = torch.matmul(S, u[t].unsqueeze(-1))                                # [H, value, 1]
            S = S * w[t].unsqueeze(1) - z * (a[t] * u[t]).unsqueeze(1) + v[t].unsqueeze(-1) * k[t].unsqueeze(1)
            o[t] = torch.matmul(S, r[t].unsqueeze(-1)).squeeze(-1)
        state[slot, :, :, :D] = S
        o = o / torch.sqrt(o.square().mean(-1, keepdim=True) + eps)
        y = o.reshape(n, W) * norm_w * torch.sigmoid(g.reshape(n, W)) * out_scale
        out[b * T:b * T + n] = y.to(out.dtype)
