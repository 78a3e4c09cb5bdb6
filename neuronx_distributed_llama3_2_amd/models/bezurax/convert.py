"""Bezurax checkpoint tensors -> the framework's parameter names.

The projections of both mixers of a layer become the rows of one in_proj (each mixer's part padded with
zero rows, so that it starts and ends 16-byte aligned for both activation types), their output
projections the columns of one o_proj; the router and the shared expert's gate the rows of one router
projection; the experts' matrices two stacks, [gate; up] and down."""

from __future__ import annotations

from typing import Dict, Sequence

import torch

from ...modules.hybrid.context import padded_rows
from .configuration import BezuraxConfig


def _pad(w: torch.Tensor, dim: int) -> torch.Tensor:
    n = padded_rows(w.shape[dim]) - w.shape[dim]
    if not n:
        return w
    shape = list(w.shape)
    shape[dim] = n
    return torch.cat([w, w.new_zeros(shape)], dim)


def _stack(parts: Sequence[torch.Tensor]) -> torch.Tensor:
    return _pad(torch.cat(list(parts), 0), 0)


def checkpoint_to_nxd(sd: Dict[str, torch.Tensor], config: BezuraxConfig) -> Dict[str, torch.Tensor]:
    out = {"model.embed_tokens.weight": sd["embed"], "model.norm.weight": sd["final.norm"]}
    for u, i in enumerate(config.unique):
        layer, src, dst = config.layers[i], f"l{i}.", f"model.layers.{u}."
        left = lambda n: sd[f"{src}mix.left.{n}"]  # noqa: E731
        right = lambda n: sd[f"{src}mix.right.{n}"]  # noqa: E731
        out[dst + "mixer.in_proj.weight"] = torch.cat(
            [_stack([left("q"), left("k")]), _stack([right(n) for n in ("r", "k", "v", "g", "a", "w1")])], 0)
        out[dst + "mixer.o_proj.weight"] = torch.cat([_pad(left("o"), 1), _pad(right("o"), 1)], 1)
        out[dst + "mixer.left.q_norm"] = left("q.norm")
        out[dst + "mixer.left.k_norm"] = left("k.norm")
        out[dst + "mixer.right.w2"] = right("w2")
        out[dst + "mixer.right.w0"] = right("w0")
        out[dst + "mixer.right.a_bias"] = right("a.b")
        out[dst + "mixer.right.out_norm"] = right("norm")
        out[dst + "norms.0"] = sd[src + "norm1"]
        m = layer.mlp
        if m is None:
            continue
        out[dst + "norms.1"] = sd[src + "norm2"]
        mlp = lambda n: sd[f"{src}mlp.{n}"]  # noqa: E731
        out[dst + "mlp.router.weight"] = _stack([mlp("router")] + ([mlp("shared.sg")] if m.shared_ff else []))
        out[dst + "mlp.gate_up"] = torch.stack([torch.cat([mlp(f"e{e}.gate"), mlp(f"e{e}.up")], 0) for e in range(m.experts)])
        out[dst + "mlp.down"] = torch.stack([mlp(f"e{e}.down") for e in range(m.experts)])
        if m.shared_ff:
            out[dst + "mlp.shared_up.weight"] = torch.cat([mlp("shared.gate"), mlp("shared.up")], 0)
            out[dst + "mlp.shared_down.weight"] = mlp("shared.down")
    return out
