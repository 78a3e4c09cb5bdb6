"""Small Golitar configurations and random weights for the tests, and the comparison they share."""

from __future__ import annotations

import json
import os

import torch
from safetensors.torch import save_file


def delta(heads=4, kv_heads=2, dim=24, vdim=40, conv=4, ff=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def attention(heads=4, kv_heads=2, dim=16, vdim=24, window=37, rot=8, base=10000.0, scaling=True, softcap=20.0, scale=0.3,
              diff=0.45, ff=96):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff, "scale": scale,
         "softcap": softcap, "mask": {"size": window} if window else None,
         "rot": {"dims": rot, "base": base,
                 "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64} if scaling else None}}
    return {"type": "attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, width=80, vocab=211, streams=2, eps=1e-5, logit_softcap=12.0):
    return {"architecture": "Golitar", "layers": layers, "width": width, "vocab": vocab, "streams": streams,
            "norm": {"eps": eps}, "logit_softcap": logit_softcap}


# the order of layers, the sizes, and what is equal or 1 differ between them
CONFIGS = {
    "mixed": config([delta(), attention(), delta(heads=3, kv_heads=3, dim=32, vdim=16, conv=2, ff=56),
                     attention(heads=6, kv_heads=2, window=5, ff=None)]),
    "attention_first": config([attention(heads=2, kv_heads=1, dim=40, vdim=64, rot=40, scaling=False, window=64),
                               delta(heads=2, kv_heads=1, dim=40, vdim=72, conv=1, ff=40)],
                              width=72, vocab=97, streams=4, eps=1e-6),
    "one_stream": config([delta(heads=1, kv_heads=1, dim=8, vdim=8, conv=3),
                          attention(heads=1, kv_heads=1, dim=10, vdim=6, rot=2, window=1),
                          attention(heads=3, kv_heads=3, dim=12, vdim=20, rot=0, window=None, softcap=60.0)],
                         width=36, vocab=53, streams=1, logit_softcap=None),
    "wide_heads": config([delta(heads=2, kv_heads=2, dim=128, vdim=96, conv=4),
                          attention(heads=2, kv_heads=2, dim=72, vdim=136, rot=64, window=90, softcap=50.0, ff=64)],
                         width=128, vocab=130, streams=3),
}


def weights(cfg, seed=0):
    """Random checkpoint tensors (bf16, as they are stored).  Everything that a mistake could leave out
    has a visible size: norms away from their neutral value, mixes that are not symmetric, keys that
    stand out among their neighbours."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0, mean=0.0: (torch.randn(*s, generator=g) * std + mean)  # noqa: E731
    W, S = cfg["width"], cfg["streams"]
    sd = {"embed": r(cfg["vocab"], W), "head": r(cfg["vocab"], W, std=2 * W ** -0.5), "final.norm": r(W, std=0.2)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        lin = lambda n, rows, cols=W, gain=1.0: sd.__setitem__(p + n, r(rows, cols, std=gain * cols ** -0.5))  # noqa: E731
        maps = 2 if layer["type"] == "attention" else 1
        lin("mix.q", (H if maps == 2 else G) * maps * D)
        lin("mix.k", G * maps * D)
        lin("mix.v", (G if maps == 2 else H) * V)
        lin("mix.o", W, H * V)
        if layer["type"] == "delta":
            for n, c in (("q", G * D), ("k", G * D), ("v", H * V)):
                sd[f"{p}mix.{n}.conv"] = r(c, m["conv"], std=0.6)
            lin("mix.b", H)
            lin("mix.a", H)
            lin("mix.g", H * V)
            sd[p + "mix.A_log"] = r(H, std=0.5, mean=-1.0)
            sd[p + "mix.dt_bias"] = r(H, std=0.5, mean=-2.0)
            sd[p + "mix.norm"] = r(V, std=0.2, mean=1.0)
        else:
            for n, c in (("q", H * 2 * D), ("k", G * 2 * D), ("v", G * V), ("o", W)):
                sd[f"{p}mix.{n}.b"] = r(c, std=0.3)
            sd[p + "mix.q.norm"] = r(D, std=0.3, mean=1.5)
            sd[p + "mix.k.norm"] = r(D, std=0.3, mean=1.5)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                sd[f"{p}mix.{n}"] = r(D, std=0.3)
        sd[p + "norm1"] = r(W, std=0.2)
        if layer["mlp"] is not None:
            lin("mlp.up", layer["mlp"]["ff"])
            lin("mlp.down", W, layer["mlp"]["ff"])
            sd[p + "norm2"] = r(W, std=0.2)
        for q in (1, 2) if layer["mlp"] is not None else (1,):
            sd[f"{p}hc{q}.in"] = r(S, std=0.4, mean=0.7)
            sd[f"{p}hc{q}.out"] = r(S, std=0.4, mean=0.8)
            sd[f"{p}hc{q}.mix"] = r(S, S, std=0.2) + torch.eye(S) * 0.8
    return {k: v.to(torch.bfloat16).contiguous() for k, v in sd.items()}


def write_model(path, cfg, sd) -> str:
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(sd, os.path.join(path, "model.safetensors"))
    return str(path)


def doubles(sd):
    return {k: v.double() for k, v in sd.items()}


def tokens(n, vocab, seed=1):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def row_errs(got, want):
    """Root mean square of the difference over that of `want`, per row."""
    got, want = got.double().cpu(), want.double()
    return (got - want).square().mean(-1).sqrt() / want.square().mean(-1).sqrt().clamp_min(1e-9)


def rel_err(got, want):
    return float(row_errs(got, want).max())


def logits_agree(got, want, dtype):
    """fp32: every row within 3e-4.  bf16: rounding alone moves single rows of these random models by up to
    a tenth, so the average is what is held small."""
    e = row_errs(got, want)
    if dtype == torch.float32:
        return float(e.max()) < 3e-4
    return float(e.mean()) < 4e-2 and float(e.max()) < 0.25
