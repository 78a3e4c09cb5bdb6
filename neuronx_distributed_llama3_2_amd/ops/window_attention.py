"""Causal attention with a sliding window, score soft-capping and one or two maps per head
(differential attention) over a per-layer ring cache (csrc/hybrid/window_attn.hip).

Cache of a layer: k [slots, G maps, cap, D], v [slots, G, cap, V]; the key of position p is entry
p % cap, so a windowed layer holds about one window of keys."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from ._ext import hybrid_ext, use_native


@dataclass(frozen=True)
class AttnSizes:
    heads: int
    kv_heads: int
    maps: int
    dim: int
    vdim: int

    @property
    def q_columns(self) -> int:
        return self.heads * self.maps * self.dim

    @property
    def k_columns(self) -> int:
        return self.kv_heads * self.maps * self.dim

    @property
    def columns(self) -> int:
        return self.q_columns + self.k_columns + self.kv_heads * self.vdim

    def as_list(self):
        return [self.heads, self.kv_heads, self.maps, self.dim, self.vdim]


@dataclass(frozen=True)
class AttnRule:
    """Score and combination constants.  window 0: every earlier token; softcap 0: none.  Two maps:
    out = out_scale * (a1 - lam a2) / sqrt(mean((a1 - lam a2)^2) + eps)."""

    scale: float
    softcap: float = 0.0
    window: int = 0
    lam: float = 0.0
    out_scale: float = 1.0
    eps: float = 0.0


def attn_prep_(buf: torch.Tensor, B: int, T: int, sizes: AttnSizes, bias: Optional[torch.Tensor],
               q_norm: Optional[torch.Tensor], k_norm: Optional[torch.Tensor], eps: float, cos_t: torch.Tensor,
               sin_t: torch.Tensor, positions: torch.Tensor, lengths: Optional[torch.Tensor],
               slots: Optional[torch.Tensor], k_cache: torch.Tensor, v_cache: torch.Tensor) -> None:
    """buf [B T, >= columns] = [q | k | v] projections of T new tokens per sequence, in place: bias, RMS
    norm of every q / k head and map, rotary turn of the pairs (2i, 2i + 1) by cos_t / sin_t
    [positions, pairs]; k and v also go to the cache of slots[b]."""
    if use_native(buf):
        hybrid_ext().attn_prep(buf, B, T, sizes.as_list(), bias, q_norm, k_norm, float(eps), cos_t, sin_t, positions,
                               lengths, slots, k_cache, v_cache)
        return
    H, G, R, D, V = sizes.as_list()
    cap, half = k_cache.shape[2], cos_t.shape[1]
    nqk = sizes.q_columns + sizes.k_columns
    for b in range(B):
        slot = int(slots[b]) if slots is not None else b
        p0 = int(positions.reshape(B, -1)[b, 0])
        n = min(T, int(lengths[b])) if lengths is not None else T
        if n == 0:
            continue
        rows = buf[b * T:b * T + n, :sizes.columns]
        x = rows.float() if bias is None else rows.float() + bias
        qk = x[:, :nqk].reshape(n, (H + G) * R, D)
        if q_norm is not None:
            w = torch.cat([q_norm.expand(H * R, D), k_norm.expand(G * R, D)])
            qk = qk / torch.sqrt(qk.square().mean(-1, keepdim=True) + eps) * w
        pos = torch.arange(p0, p0 + n).clamp(max=cos_t.shape[0] - 1)
        c, s = cos_t[pos].unsqueeze(1), sin_t[pos].unsqueeze(1)
        u, w2 = qk[..., 0:2 * half:2], qk[..., 1:2 * half:2]
        qk = qk.clone()
        turned = torch.stack([u * c - w2 * s, w2 * c + u * s], -1).flatten(-2)
        qk[..., :2 * half] = turned
        rows[:, :nqk] = qk.reshape(n, -1).to(buf.dtype)
        rows[:, nqk:] = x[:, nqk:].to(buf.dtype)
        for t in range(max(0, n - cap), n):
            e = (p0 + t) % cap
            k_cache[slot, :, e] = rows[t, sizes.q_columns:nqk].view(G * R, D)
            v_cache[slot, :, e] = rows[t, nqk:].view(G, V)


def window_attention(buf: torch.Tensor, B: int, T: int, sizes: AttnSizes, rule: AttnRule, positions: torch.Tensor,
                     lengths: Optional[torch.Tensor], slots: Optional[torch.Tensor], k_cache: torch.Tensor,
                     v_cache: torch.Tensor, prompt: bool, fused: bool = True) -> torch.Tensor:
    """Attention of the queries in buf (after attn_prep_): over the tokens of this step when they start
    at position 0 (`prompt`), else over the cache (a ring that wraps must hold window + T - 1 keys).  Returns [B T, H V] (padding rows are zero).
    fused: the matrix-core prompt kernel and the split decode kernel where the sizes allow (bf16)."""
    H, G, R, D, V = sizes.as_list()
    y = torch.empty((B * T, H * V), dtype=buf.dtype, device=buf.device)
    if use_native(buf):
        hybrid_ext().window_attn(buf, B, T, sizes.as_list(), rule.scale, rule.softcap, rule.window, rule.lam,
                                 rule.out_scale, rule.eps, positions, lengths, slots, k_cache, v_cache, y, prompt, fused)
        return y
    y.zero_()
    cap = k_cache.shape[2]
    if not prompt and T > cap:
        raise ValueError(f"{T} new tokens do not fit a ring of {cap}")
    for b in range(B):
        slot = int(slots[b]) if slots is not None else b
        p0 = int(positions.reshape(B, -1)[b, 0])
        n = min(T, int(lengths[b])) if lengths is not None else T
        if n == 0:
            continue
        rows = buf[b * T:b * T + n]
        q = rows[:, :sizes.q_columns].reshape(n, H, R, D).float()
        lo = max(0, p0 - rule.window + 1) if rule.window > 0 else 0
        keys = torch.arange(0 if prompt else lo, p0 + n)
        if prompt:
            k = rows[:, sizes.q_columns:sizes.q_columns + sizes.k_columns].reshape(n, G, R, D).float()
            v = rows[:, sizes.q_columns + sizes.k_columns:sizes.columns].reshape(n, G, V).float()
        else:
            k = k_cache[slot][:, keys % cap].float().view(G, R, -1, D).permute(2, 0, 1, 3)
            v = v_cache[slot][:, keys % cap].float().transpose(0, 1)
        qpos = torch.arange(p0, p0 + n)
        seen = keys[None, :] <= qpos[:, None]
        if rule.window > 0:
            seen &= qpos[:, None] - keys[None, :] < rule.window
        k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
        s = torch.einsum("nhrd,khrd->hrnk", q, k) * rule.scale
        if rule.softcap > 0:
            s = rule.softcap * torch.tanh(s / rule.softcap)
        a = torch.einsum("hrnk,khv->nhrv", torch.softmax(s.masked_fill(~seen, float("-inf")), -1), v)
        o = a[:, :, 0]
        if R == 2:
            o = o - rule.lam * a[:, :, 1]
            o = o / torch.sqrt(o.square().mean(-1, keepdim=True) + rule.eps) * rule.out_scale
        y[b * T:b * T + n] = o.reshape(n, H * V).to(y.dtype)
    return y


def attn_decode(buf: torch.Tensor, sizes: AttnSizes, rule: AttnRule, bias: Optional[torch.Tensor],
                q_norm: Optional[torch.Tensor], k_norm: Optional[torch.Tensor], eps: float, cos_t: torch.Tensor,
                sin_t: torch.Tensor, positions: torch.Tensor, slots: Optional[torch.Tensor], k_cache: torch.Tensor,
                v_cache: torch.Tensor, tickets: torch.Tensor) -> torch.Tensor:
    """attn_prep_ and window_attention for one new token per sequence in one launch
    (csrc/hybrid/window_attn_decode.hip); buf [B, >= columns] is left as it is.  tickets: int32 zeros,
    B * heads of them, left at zero."""
    B = buf.shape[0]
    if use_native(buf):
        y = torch.empty((B, sizes.heads * sizes.vdim), dtype=buf.dtype, device=buf.device)
        hybrid_ext().attn_decode(buf, sizes.as_list(), bias, q_norm, k_norm, float(eps), cos_t, sin_t, rule.scale,
                                 rule.softcap, rule.window, rule.lam, rule.out_scale, rule.eps, positions, slots,
                                 k_cache, v_cache, tickets, y)
        return y
    buf = buf.clone()
    attn_prep_(buf, B, 1, sizes, bias, q_norm, k_norm, eps, cos_t, sin_t, positions, None, slots, k_cache, v_cache)
    return window_attention(buf, B, 1, sizes, rule, positions, None, slots, k_cache, v_cache, False)
