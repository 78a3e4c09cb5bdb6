"""Residual sum and grouped RMS norms (csrc/hybrid/group_norm.hip): the step between two layers of a
decoder whose sublayers read the same residual side by side."""

from __future__ import annotations

from typing import List, Optional, Sequence

import torch

from ._ext import hybrid_ext, use_native


def residual_norms(x: torch.Tensor, norms: Sequence[torch.Tensor], eps: float, groups: int = 1,
                   embed: Optional[torch.Tensor] = None, ids: Optional[torch.Tensor] = None,
                   adds: Sequence[torch.Tensor] = (), pairs: Optional[torch.Tensor] = None,
                   inverse: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None, store: bool = True,
                   dtype: Optional[torch.dtype] = None) -> List[torch.Tensor]:
    """One launch on the residual x [M, W] fp32 (updated in place when `store`):

      x_m = x_m (or embed[ids[m]]) + sum of adds[.][m] + sum_j pairs[inverse[m, j]]
      h_n = x / sqrt(mean of x^2 over each of `groups` equal parts + eps) * norms[n]

    for at most two adds and two norms (fp32 [W]).  pairs [P, W], inverse int32 [M, k]: outputs of
    (token, choice) pairs and where each is (None: in order, P / M for each row).  rows [R] (int64): only these rows, read-only (store=False).
    Returns the normalised rows in `dtype` (that of the adds / embed)."""
    M, W = x.shape
    src = embed if embed is not None else (adds[0] if adds else pairs)
    dtype = dtype or (src.dtype if src is not None else torch.bfloat16)
    store = store and rows is None
    R = M if rows is None else rows.numel()
    if use_native(x):
        hs = [torch.empty((R, W), dtype=dtype, device=x.device) for _ in norms]
        hybrid_ext().residual_norms(x, embed, ids, list(adds), pairs, inverse, list(norms), float(eps), groups, hs, rows, store)
        return hs
    y = x
    if embed is not None:
        ok = (ids >= 0) & (ids < embed.shape[0])
        y = embed[ids.clamp(0, embed.shape[0] - 1)].float() * ok.unsqueeze(-1)
    for a in adds:
        y = y + a.float()
    if pairs is not None:
        y = y + (pairs[inverse.long()] if inverse is not None else pairs.view(M, -1, W)).float().sum(1)
    if store:
        x.copy_(y)
    if rows is not None:
        y = y[rows]
    p = y.reshape(R, groups, W // groups)
    n = (p / torch.sqrt(p.square().mean(-1, keepdim=True) + eps)).reshape(R, W)
    return [(n * w).to(dtype) for w in norms]
