"""Golitar checkpoint tensors -> the framework's parameter names.

A delta layer's projections (q, k, v, output gate, write strength, decay) become the rows of one
in_proj, an attention layer's q / k / v the rows of one qkv_proj; the row count is padded with zero
rows so that every row of the projection buffer is 16-byte aligned for both activation types."""

from __future__ import annotations

from typing import Dict

import torch

from ...modules.hybrid.context import padded_rows
from .configuration import GolitarConfig

def _stack(parts) -> torch.Tensor:
    w = torch.cat(list(parts), 0)
    pad = padded_rows(w.shape[0]) - w.shape[0]
    return torch.cat([w, w.new_zeros((pad,) + tuple(w.shape[1:]))], 0) if pad else w


def checkpoint_to_nxd(sd: Dict[str, torch.Tensor], config: GolitarConfig) -> Dict[str, torch.Tensor]:
    out = {"model.embed_tokens.weight": sd["embed"], "model.norm.weight": sd["final.norm"], "lm_head.weight": sd["head"]}
    for i, layer in enumerate(config.layers):
        src, dst = f"l{i}.", f"model.layers.{i}."
        mix = lambda n: sd[f"{src}mix.{n}"]  # noqa: E731
        out[dst + "mixer.o_proj.weight"] = mix("o")
        if layer.type == "delta":
            out[dst + "mixer.in_proj.weight"] = _stack(mix(n) for n in ("q", "k", "v", "g", "b", "a"))
            out[dst + "mixer.conv"] = torch.cat([mix(n + ".conv") for n in ("q", "k", "v")], 0).t().contiguous()
            out[dst + "mixer.out_norm"] = mix("norm")
            out[dst + "mixer.a_log"] = mix("A_log")
            out[dst + "mixer.dt_bias"] = mix("dt_bias")
        else:
            out[dst + "mixer.qkv_proj.weight"] = _stack(mix(n) for n in ("q", "k", "v"))
            out[dst + "mixer.qkv_bias"] = torch.cat([mix(n + ".b") for n in ("q", "k", "v")], 0)
            out[dst + "mixer.o_bias"] = mix("o.b")
            out[dst + "mixer.q_norm"] = mix("q.norm")
            out[dst + "mixer.k_norm"] = mix("k.norm")
            for n in ("lq1", "lk1", "lq2", "lk2"):
                out[f"{dst}mixer.{n}"] = mix(n)
        if layer.ff is not None:
            out[dst + "mlp.up_proj.weight"] = sd[src + "mlp.up"]
            out[dst + "mlp.down_proj.weight"] = sd[src + "mlp.down"]
        for q in (1, 2) if layer.ff is not None else (1,):
            out[f"{dst}norms.{q - 1}"] = sd[f"{src}norm{q}"]
            for theirs, ours in (("in", "read"), ("mix", "mix"), ("out", "write")):
                out[f"{dst}hyper.{q - 1}.{ours}"] = sd[f"{src}hc{q}.{theirs}"]
    return out
