"""Hyper-connections (csrc/hybrid/hyper_conn.hip): S residual streams [M, S, W] in fp32, mixed around
every sublayer, and the small element-wise operations of the decoders that use them."""

from __future__ import annotations

from typing import Optional

import torch

from ._ext import hybrid_ext, use_native


def hyper_step(streams: torch.Tensor, y: Optional[torch.Tensor] = None, y_bias: Optional[torch.Tensor] = None,
               mix: Optional[torch.Tensor] = None, write: Optional[torch.Tensor] = None,
               read: Optional[torch.Tensor] = None, norm_w: Optional[torch.Tensor] = None, eps: float = 0.0,
               embed: Optional[torch.Tensor] = None, ids: Optional[torch.Tensor] = None,
               rows: Optional[torch.Tensor] = None, store: bool = True, dtype: Optional[torch.dtype] = None):
    """One launch between two sublayers, on streams [M, S, W] fp32 (updated in place when `store`):

      x_t = sum_s mix[s, t] x_s + write[t] (y + y_bias)     (with y [M, W], the last sublayer's output)
      h   = (1 + norm_w) * rms_normalise(sum_s read[s] x_s) (with read: the next sublayer's input)

    embed / ids: the streams start as embed[ids] (their old contents are ignored).  rows [R] (int64):
    only these rows, read-only (store=False).  Returns h [R, W] in `dtype` (that of y / embed), or None
    without `read`."""
    M, S, W = streams.shape
    src = y if y is not None else embed
    dtype = dtype or (src.dtype if src is not None else torch.bfloat16)
    store = store and rows is None
    if use_native(streams):
        h = None
        if read is not None:
            h = torch.empty((M if rows is None else rows.numel(), W), dtype=dtype, device=streams.device)
        hybrid_ext().hyper_step(streams, embed, ids, y, y_bias, mix, write, read, norm_w, float(eps), h, rows, store)
        return h
    x = streams
    if embed is not None:
        ok = (ids >= 0) & (ids < embed.shape[0])
        e = embed[ids.clamp(0, embed.shape[0] - 1)].float() * ok.unsqueeze(-1)
        x = e.unsqueeze(1).expand(M, S, W)
    if y is not None:
        yf = y.float() if y_bias is None else y.float() + y_bias
        x = torch.einsum("st,msw->mtw", mix, x) + write[None, :, None] * yf.unsqueeze(1)
    if store:
        streams.copy_(x)
    if read is None:
        return None
    if rows is not None:
        x = x[rows]
    u = torch.einsum("s,msw->mw", read, x)
    return (u / torch.sqrt((u * u).mean(-1, keepdim=True) + eps) * (1.0 + norm_w)).to(dtype)


def relu_squared(x: torch.Tensor) -> torch.Tensor:
    if use_native(x):
        x = x.contiguous()
        y = torch.empty_like(x)
        hybrid_ext().relu_squared(x, y)
        return y
    return torch.relu(x.float()).square().to(x.dtype)


def softcap_(x: torch.Tensor, cap: float) -> torch.Tensor:
    """x = cap tanh(x / cap) in place (contiguous fp32)."""
    if use_native(x):
        hybrid_ext().softcap_(x, float(cap))
        return x
    return x.copy_(cap * torch.tanh(x / cap))


FUSED_ROWS = 4               # most rows the fused decode projections take
FUSED_NORM_ELEMENTS = 24576  # most elements of the rows they normalise (48 KB of LDS)

_EPI = {"store": 0, "relu2": 1, "f32": 2, "streams": 3}


def decode_linear(w: torch.Tensor, x: Optional[torch.Tensor] = None, u: Optional[torch.Tensor] = None,
                  norm_w: Optional[torch.Tensor] = None, eps: float = 0.0, epilogue: str = "store", cap: float = 0.0,
                  alpha: float = 1.0):
    """epilogue(x w^T) for a few rows in one launch (csrc/hybrid/gemv_hyper.hip, GPU, bf16 weights): x
    bf16 [M, K], or u fp32 [M, K], normalised as hyper_step does on the way in.  "store": bf16, "relu2":
    bf16 squared ReLU, "f32": fp32 alpha y, with cap > 0 cap tanh(alpha y / cap)."""
    M = (x if x is not None else u).shape[0]
    y = torch.empty((M, w.shape[0]), dtype=torch.float32 if epilogue == "f32" else torch.bfloat16, device=w.device)
    hybrid_ext().gemv_hyper(_EPI[epilogue], x, u, norm_w, float(eps), w, y, float(cap), alpha=float(alpha))
    return y


def decode_linear_into_streams(w: torch.Tensor, x: torch.Tensor, streams: torch.Tensor, bias: Optional[torch.Tensor],
                               mix: torch.Tensor, write: torch.Tensor, read: torch.Tensor) -> torch.Tensor:
    """The output projection of a sublayer with the write into the streams as its epilogue (in place);
    returns u [M, W] fp32, what the next sublayer reads before its norm."""
    un = torch.empty((x.shape[0], w.shape[0]), dtype=torch.float32, device=w.device)
    hybrid_ext().gemv_hyper(_EPI["streams"], x, None, None, 0.0, w, None, 0.0, streams, bias, mix, write, read, un)
    return un
