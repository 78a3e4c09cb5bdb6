"""Small Bezurax configurations and random weights for the tests."""

from __future__ import annotations

import torch


def mixer(heads=4, kv_heads=2, dim=16, scale=0.4, window=37, pool=6, rheads=3, rdim=20, left_scale=0.7, right_scale=1.2):
    return {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
                     "mask": {"size": window, "pool": pool}},
            "left_scale": left_scale, "right": {"heads": rheads, "dim": rdim}, "right_scale": right_scale}


def moe(experts=6, top=2, ff=24, limit=1.2, scale=1.7, groups=(3, 2), shared_ff=40, shared_limit=0.8):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
         "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups[0], "keep": groups[1]}}}
    if shared_ff:
        m["shared"] = {"ff": shared_ff, "limit": shared_limit}
    return m


def layer(mix, mlp, weights_of=None):
    d = {"type": "parallel", "mixer": mix, "mlp": mlp}
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


def config(layers, width=72, vocab=211, eps=1e-5, groups=3, logit_scale=0.8):
    return {"architecture": "Bezurax", "layers": layers, "width": width, "vocab": vocab,
            "norm": {"eps": eps, "groups": groups}, "logit_scale": logit_scale}


# the order of layers, the sizes, the limits and what is equal or 1 differ between them
_A = layer(mixer(), moe())
_B = layer(mixer(heads=3, kv_heads=3, dim=24, window=20, pool=9, rheads=2, rdim=40), None)
CONFIGS = {
    "mixed": config([_A, _B, layer(_A["mixer"], _A["mlp"], 0),
                     layer(mixer(heads=6, kv_heads=1, dim=8, window=3, pool=5, rheads=1, rdim=33, scale=1.0),
                           moe(experts=5, top=5, ff=17, groups=(1, 1), shared_ff=0)),
                     layer(_B["mixer"], None, 1)]),
    # nothing grouped, a block a token, one expert of its group
    "plain": config([layer(mixer(heads=2, kv_heads=1, dim=10, window=1, pool=1, rheads=2, rdim=9, left_scale=1.0, right_scale=1.0),
                           moe(experts=4, top=1, ff=16, scale=1.0, groups=(4, 2), shared_ff=8, shared_limit=3.0))],
                    width=36, vocab=53, groups=1, logit_scale=1.0, eps=1e-6),
    "one_expert": config([layer(mixer(heads=1, kv_heads=1, dim=8, window=64, pool=16, rheads=1, rdim=8),
                                moe(experts=1, top=1, ff=8, groups=(1, 1))),
                          layer(mixer(heads=4, kv_heads=4, dim=40, window=65, pool=64, rheads=4, rdim=16),
                                moe(experts=12, top=6, ff=32, limit=0.5, groups=(2, 1)))],
                         width=64, vocab=97, groups=2),
    "wide_heads": config([layer(mixer(heads=4, kv_heads=2, dim=72, window=90, pool=12, rheads=2, rdim=128, scale=0.2),
                                moe(experts=8, top=3, ff=64, groups=(4, 3), shared_ff=64)),
                          layer(mixer(heads=2, kv_heads=2, dim=128, window=33, pool=7, rheads=3, rdim=64, scale=0.1),
                                moe(experts=16, top=4, ff=40, groups=(4, 2), shared_ff=32))],
                         width=128, vocab=130, groups=4),
    "large_heads": config([layer(mixer(heads=2, kv_heads=1, dim=136, window=24, pool=8, rheads=1, rdim=136, scale=0.1),
                                 moe(experts=4, top=2, ff=32, groups=(2, 1)))], width=64, vocab=67, groups=8),
}
RANKS = {"mixed": 7, "plain": 1, "one_expert": 16, "wide_heads": 24, "large_heads": 70, "long": 5}


def weights(cfg, seed=0, rank=7):
    """Random checkpoint tensors (bf16, as they are stored).  Everything that a mistake could leave out has a
    visible size: norms and biases away from their neutral value, activations beyond the limits, experts
    whose scores are far apart, keys that are not lost among their neighbours."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0, mean=0.0: torch.randn(*s, generator=g) * std + mean  # noqa: E731
    W = cfg["width"]
    sd = {"embed": r(cfg["vocab"], W), "final.norm": r(W, std=0.2, mean=1.0)}
    for i, l in enumerate(cfg["layers"]):
        if "weights_of" in l:
            continue
        p, a, d = f"l{i}.", l["mixer"]["left"], l["mixer"]["right"]
        lin = lambda n, rows, cols=W, gain=1.0: sd.__setitem__(p + n, r(rows, cols, std=gain * cols ** -0.5))  # noqa: E731
        nq, nk, n = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], d["heads"] * d["dim"]
        sd[p + "norm1"] = r(W, std=0.2, mean=1.0)
        lin("mix.left.q", nq)
        lin("mix.left.k", nk)
        lin("mix.left.o", W, nq)
        sd[p + "mix.left.q.norm"] = r(nq, std=0.3, mean=1.2)
        sd[p + "mix.left.k.norm"] = r(nk, std=0.3, mean=1.2)
        for t in ("r", "k", "v", "g", "a"):
            lin(f"mix.right.{t}", n)
        lin("mix.right.o", W, n)
        lin("mix.right.w1", rank)
        lin("mix.right.w2", n, rank, 1.5)
        sd[p + "mix.right.w0"] = r(n, std=1.0, mean=-2.0)
        sd[p + "mix.right.a.b"] = r(n, std=0.5)
        sd[p + "mix.right.norm"] = r(n, std=0.2, mean=1.0)
        m = l["mlp"]
        if m is None:
            continue
        sd[p + "norm2"] = r(W, std=0.2, mean=1.0)
        lin("mlp.router", m["router"]["experts"], gain=1.5)
        for pre, f in [(f"mlp.e{e}.", m["expert"]["ff"]) for e in range(m["router"]["experts"])] + \
                      ([("mlp.shared.", m["shared"]["ff"])] if m.get("shared") else []):
            lin(pre + "gate", f)
            lin(pre + "up", f)
            lin(pre + "down", W, f)
        if m.get("shared"):
            lin("mlp.shared.sg", 1)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in sd.items()}
