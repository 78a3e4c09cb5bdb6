"""Causal attention with a sliding window and pooled blocks (csrc/hybrid/pooled_attn.hip and the windowed
kernels): a query sees the last `window` tokens and, in the same softmax, one key and value for every
block of `pool` tokens that has left its window -- the means of the block's keys and values.  Queries and
keys are normalised over the whole projection, values are the keys as projected, there are no positions.

Cache of a layer: k, v [slots, G, cap, D] rings of recent tokens (position p in entry p % cap) and
pk, pv [slots, G, blocks, D], block b in entry b, written by the step that brings the block's last token."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from ._ext import hybrid_ext, use_native


@dataclass(frozen=True)
class PooledSizes:
    heads: int
    kv_heads: int
    dim: int

    @property
    def q_columns(self) -> int:
        return self.heads * self.dim

    @property
    def columns(self) -> int:    # q | k
        return (self.heads + self.kv_heads) * self.dim

    def as_list(self):
        return [self.heads, self.kv_heads, self.dim]


@dataclass(frozen=True)
class PooledRule:
    scale: float
    window: int
    pool: int
    eps: float            # of the query / key norm


def blocks_seen(pos: int, rule: PooledRule) -> int:
    """Pooled blocks that the query at `pos` sees."""
    return max(0, (pos - rule.window + 1) // rule.pool)


def _span(b, B, T, positions, lengths, slots):
    slot = int(slots[b]) if slots is not None else b
    p0 = int(positions.reshape(B, -1)[b, 0])
    return slot, p0, (min(T, int(lengths[b])) if lengths is not None else T)


def pooled_prep_(buf: torch.Tensor, B: int, T: int, sizes: PooledSizes, rule: PooledRule, q_norm: torch.Tensor,
                 k_norm: torch.Tensor, positions: torch.Tensor, lengths: Optional[torch.Tensor],
                 slots: Optional[torch.Tensor], cache: Dict[str, torch.Tensor], prompt: bool) -> torch.Tensor:
    """buf [B T, >= columns] = [q | k] projections of T new tokens per sequence: q is normalised in place, k
    stays as projected (the values); returns the normalised keys [B T, G D].  Keys and values go to the
    rings of slots[b], the means of the blocks that these tokens complete to its pooled entries."""
    H, G, D = sizes.as_list()
    kn = torch.empty((B * T, G * D), dtype=buf.dtype, device=buf.device)
    kc, vc, pk, pv = cache["k"], cache["v"], cache["pk"], cache["pv"]
    if use_native(buf):
        hybrid_ext().pooled_prep(buf, kn, B, T, sizes.as_list(), q_norm, k_norm, rule.eps, rule.pool, positions, lengths, slots,
                                 kc, vc, pk, pv, prompt)
        return kn
    cap, nq = kc.shape[2], sizes.q_columns
    if not prompt and T + max(rule.pool, rule.window) - 1 > cap and cap < int(positions.max()) + 1:
        raise ValueError(f"{T} new tokens do not fit a ring of {cap}")
    kn.zero_()
    for b in range(B):
        slot, p0, n = _span(b, B, T, positions, lengths, slots)
        if n == 0:
            continue
        rows = buf[b * T:b * T + n]
        for part, w in ((rows[:, :nq], q_norm), (rows[:, nq:sizes.columns], k_norm)):
            x = part.float()
            x = (x / torch.sqrt(x.square().mean(-1, keepdim=True) + rule.eps) * w).to(buf.dtype)
            if part.shape[1] == nq and w is q_norm:
                part.copy_(x)
            else:
                kn[b * T:b * T + n] = x
        k = kn[b * T:b * T + n].view(n, G, D)
        v = rows[:, nq:sizes.columns].reshape(n, G, D)
        for t in range(max(0, n - cap), n):
            kc[slot, :, (p0 + t) % cap], vc[slot, :, (p0 + t) % cap] = k[t], v[t]
        for blk in range(p0 // rule.pool, (p0 + n) // rule.pool):   # blocks that end within this step
            p = torch.arange(blk * rule.pool, (blk + 1) * rule.pool)
            kk = k[p - p0].transpose(0, 1) if prompt else kc[slot][:, p % cap]
            vv = v[p - p0].transpose(0, 1) if prompt else vc[slot][:, p % cap]
            if blk < pk.shape[2]:
                pk[slot, :, blk], pv[slot, :, blk] = kk.float().mean(1).to(pk.dtype), vv.float().mean(1).to(pv.dtype)
    return kn


def pooled_attention(buf: torch.Tensor, kn: torch.Tensor, B: int, T: int, sizes: PooledSizes, rule: PooledRule,
                     positions: torch.Tensor, lengths: Optional[torch.Tensor], slots: Optional[torch.Tensor],
                     cache: Dict[str, torch.Tensor], prompt: bool, out: torch.Tensor, out_scale: float = 1.0,
                     fused: bool = True) -> None:
    """out [B T, H D] = out_scale * attention of the queries in buf (after pooled_prep_), over this step's
    tokens when they start at position 0 (`prompt`), else over the rings; padding rows are zero.  fused: the
    matrix-core prompt kernel where the sizes allow (bf16)."""
    H, G, D = sizes.as_list()
    kc, vc, pk, pv = cache["k"], cache["v"], cache["pk"], cache["pv"]
    if use_native(buf):
        hybrid_ext().pooled_attn(buf, kn, B, T, sizes.as_list(), rule.scale, rule.window, rule.pool, positions, lengths, slots,
                                 kc, vc, pk, pv, out, float(out_scale), prompt, fused)
        return
    out.zero_()
    cap = kc.shape[2]
    for b in range(B):
        slot, p0, n = _span(b, B, T, positions, lengths, slots)
        if n == 0:
            continue
        q = buf[b * T:b * T + n, :sizes.q_columns].reshape(n, H, D).float()
        keys = torch.arange(0 if prompt else max(0, p0 - rule.window + 1), p0 + n)
        if prompt:
            k = kn[b * T:b * T + n].view(n, G, D).float()
            v = buf[b * T:b * T + n, sizes.q_columns:sizes.columns].reshape(n, G, D).float()
        else:
            k, v = (c[slot][:, keys % cap].float().transpose(0, 1) for c in (kc, vc))
        nb = blocks_seen(p0 + n - 1, rule)
        k = torch.cat([pk[slot][:, :nb].float().transpose(0, 1), k]).repeat_interleave(H // G, 1)
        v = torch.cat([pv[slot][:, :nb].float().transpose(0, 1), v]).repeat_interleave(H // G, 1)
        qpos = torch.arange(p0, p0 + n)[:, None]
        seen = torch.cat([(torch.arange(nb)[None] + 1) * rule.pool - 1 <= qpos - rule.window,
                          (keys[None] <= qpos) & (qpos - keys[None] < rule.window)], 1)
        s = torch.einsum("nhd,khd->hnk", q, k) * rule.scale
        a = torch.softmax(s.masked_fill(~seen, float("-inf")), -1)
        out[b * T:b * T + n] = (torch.einsum("hnk,khd->nhd", a, v) * out_scale).reshape(n, H * D).to(out.dtype)


def pooled_decode(buf: torch.Tensor, sizes: PooledSizes, rule: PooledRule, q_norm: torch.Tensor, k_norm: torch.Tensor,
                  positions: torch.Tensor, slots: Optional[torch.Tensor], cache: Dict[str, torch.Tensor], out: torch.Tensor,
                  out_scale: float = 1.0) -> None:
    """pooled_prep_ and pooled_attention for one new token per sequence in one launch
    (csrc/hybrid/window_attn_decode.hip); buf [B, >= columns] is left as it is.  cache["tickets"]: int32
    zeros, B heads of them, left at zero."""
    B = buf.shape[0]
    if use_native(buf):
        hybrid_ext().pooled_decode(buf, sizes.as_list(), q_norm, k_norm, rule.eps, rule.scale, rule.window, rule.pool, positions,
                                   slots, cache["k"], cache["v"], cache["pk"], cache["pv"], cache["tickets"], out, float(out_scale))
        return
    buf = buf.clone()
    kn = pooled_prep_(buf, B, 1, sizes, rule, q_norm, k_norm, positions, None, slots, cache, False)
    pooled_attention(buf, kn, B, 1, sizes, rule, positions, None, slots, cache, False, out, out_scale)
