"""Mixer "differential attention": two softmax maps per head over the same values, subtracted; with
biases, per-head q / k norms, interleaved partial rotary positions, soft-capped scores and a sliding
window."""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn as nn

from ... import ops
from ...ops.rope import llama3_inv_freq
from ...ops.window_attention import AttnRule, AttnSizes
from .context import StepContext, linear, padded_rows, small

# new tokens a decode step may bring beyond the first without pushing a key that one of them still
# sees out of a windowed layer's ring
RING_SLACK = 15


def interleaved_rope_tables(dims: int, base: float, max_pos: int, factor: Optional[float] = None, low: float = 1.0,
                            high: float = 4.0, original: float = 8192.0, device=None):
    """cos / sin [max_pos, dims / 2] fp32; angles in float64, so a table entry is the rounded exact value."""
    f = llama3_inv_freq(dims, base, factor, low, high, original, dtype=torch.float64)
    a = torch.outer(torch.arange(max_pos, dtype=torch.float64), f)
    return a.cos().float().contiguous().to(device), a.sin().float().contiguous().to(device)


class DifferentialAttentionMixer(nn.Module):
    in_epilogue = "store"
    recurrent = False

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, diff: float, scale: float,
                 rot, eps: float, softcap: float = 0.0, window: int = 0, dtype=torch.bfloat16, device=None):
        super().__init__()
        self.sizes = AttnSizes(heads, kv_heads, 2, dim, vdim)
        self.diff, self.scale, self.softcap, self.window, self.eps, self.rot = diff, scale, softcap, window, eps, rot
        n = self.sizes.columns
        self.qkv_proj = nn.Linear(width, padded_rows(n), bias=False, dtype=dtype, device=device)
        self.qkv_bias = small(n, device=device)   # added in fp32 by ops.attn_prep_
        self.q_norm = small(dim, device=device)
        self.k_norm = small(dim, device=device)
        for name in ("lq1", "lk1", "lq2", "lk2"):
            setattr(self, name, small(dim, device=device))
        self.o_proj = nn.Linear(heads * vdim, width, bias=False, dtype=dtype, device=device)
        self.o_bias = small(width, device=device)   # added in fp32 when the residual streams are updated
        self._rule: Optional[AttnRule] = None
        self._tables = None

    @torch.no_grad()
    def reset_parameters(self) -> None:
        for p in (self.qkv_bias, self.o_bias):
            p.zero_()
        for p in (self.q_norm, self.k_norm):
            p.fill_(1.0)
        for name in ("lq1", "lk1", "lq2", "lk2"):
            getattr(self, name).normal_(0.0, 0.1)
        self._rule = None

    def weights_changed(self) -> None:
        self._rule = None

    @property
    def rule(self) -> AttnRule:
        """Constants of the attention kernels; lambda is one number per layer, read from its vectors once
        per weight load (never inside a graph capture)."""
        if self._rule is None:
            dot = lambda a, b: torch.exp((a.double() * b.double()).sum())  # noqa: E731
            lam = float(dot(self.lq1, self.lk1) - dot(self.lq2, self.lk2)) + self.diff
            self._rule = AttnRule(self.scale, self.softcap, self.window, lam, 1.0 - self.diff, self.eps)
        return self._rule

    def prepare(self, max_pos: int, device) -> None:
        """Rotary tables for positions below max_pos, and the constants of `rule`."""
        if self._tables is None or self._tables[0].shape[0] < max_pos or self._tables[0].device != torch.device(device):
            r = self.rot
            self._tables = interleaved_rope_tables(r.dims, r.base, max_pos, r.factor, r.low, r.high, r.original, device)
        _ = self.rule

    def cache_tensors(self, slots: int, max_len: int, dtype: torch.dtype, device) -> Dict[str, torch.Tensor]:
        s, cap = self.sizes, max_len
        if self.window:
            cap = min(max_len, (self.window + RING_SLACK + 63) // 64 * 64)
        z = lambda *shape: torch.zeros(shape, dtype=dtype, device=device)  # noqa: E731
        return {"k": z(slots, s.kv_heads * s.maps, cap, s.dim), "v": z(slots, s.kv_heads, cap, s.vdim),
                "tickets": torch.zeros(slots * s.heads, dtype=torch.int32, device=device)}

    def max_new_tokens(self, cache: Dict[str, torch.Tensor], max_len: int) -> int:
        """Tokens one decode step may bring: the ring must still hold what the first of them sees."""
        cap = cache["k"].shape[2]
        return max_len if cap >= max_len else cap - self.window + 1

    @property
    def in_linear(self) -> nn.Linear:
        return self.qkv_proj

    @property
    def out_linear(self) -> nn.Linear:
        return self.o_proj

    def core(self, buf: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext) -> torch.Tensor:
        """From the input projection's output (whose q / k / v it may overwrite) to the output projection's
        input."""
        cos_t, sin_t = self._tables
        if ctx.fused and ctx.T == 1 and not ctx.prompt and ctx.lengths is None:
            return ops.attn_decode(buf, self.sizes, self.rule, self.qkv_bias, self.q_norm, self.k_norm, self.eps, cos_t,
                                   sin_t, ctx.positions, ctx.slots, cache["k"], cache["v"], cache["tickets"])
        ops.attn_prep_(buf, ctx.B, ctx.T, self.sizes, self.qkv_bias, self.q_norm, self.k_norm, self.eps, cos_t, sin_t,
                       ctx.positions, ctx.lengths, ctx.slots, cache["k"], cache["v"])
        return ops.window_attention(buf, ctx.B, ctx.T, self.sizes, self.rule, ctx.positions, ctx.lengths, ctx.slots,
                                    cache["k"], cache["v"], ctx.prompt, ctx.fused)

    def forward(self, h: torch.Tensor, cache: Dict[str, torch.Tensor], ctx: StepContext) -> torch.Tensor:
        return linear(self.core(linear(h, self.qkv_proj), cache, ctx), self.o_proj)
