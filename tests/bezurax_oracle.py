"""Plain, slow implementation of the Bezurax design, one function per mechanism (the tests' oracle).

Written from the design's equations, one token / one head at a time wherever that is the equation's
own form, and sharing no code with the package.  Everything runs in the dtype of its inputs (the tests
use float64).  `weights` is a dict of tensors under the checkpoint's tensor names, `cfg` the parsed
config.json.
"""

from __future__ import annotations

import math

import torch


def rms_normalise(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def grouped_norm(x, w, eps, groups):
    """Each of `groups` equal consecutive parts of the last dimension over its own root mean square."""
    parts = x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups))
    return rms_normalise(parts, eps).reshape(x.shape) * w


# ------------------------------------------------------------------ attention: window and pooled blocks
def blocks_seen(i, window, pool):
    """Blocks (of `pool` tokens, from the sequence's start) that query i sees: those whose last token has
    left its window."""
    n = 0
    while (n + 1) * pool - 1 <= i - window:
        n += 1
    return n


def pooled_attention(q, k, v, scale, window, pool):
    """One head: q, k [T, D], v [T, V] -> [T, V].  Query i: tokens j with 0 <= i - j < window and, in the same
    softmax, the means of the keys and values of each block it sees."""
    T = q.shape[0]
    nb = T // pool
    kb = torch.stack([k[b * pool:(b + 1) * pool].mean(0) for b in range(nb)]) if nb else k[:0]
    vb = torch.stack([v[b * pool:(b + 1) * pool].mean(0) for b in range(nb)]) if nb else v[:0]
    out = torch.zeros(T, v.shape[1], dtype=v.dtype)
    for i in range(T):
        lo, n = max(0, i - window + 1), blocks_seen(i, window, pool)
        keys = torch.cat([kb[:n], k[lo:i + 1]])
        values = torch.cat([vb[:n], v[lo:i + 1]])
        s = (keys @ q[i]) * scale
        e = torch.exp(s - s.max())
        out[i] = (e / e.sum()) @ values
    return out


def attention_mixer(h, m, W, pre, eps):
    """h [T, width] -> [T, width]: norms over whole projections, values = keys as projected, no positions."""
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q, k = h @ W[pre + "q"].T, h @ W[pre + "k"].T
    v = k.view(T, G, D)
    q = (rms_normalise(q, eps) * W[pre + "q.norm"]).view(T, H, D)
    k = (rms_normalise(k, eps) * W[pre + "k.norm"]).view(T, G, D)
    heads = []
    for i in range(H):
        g = i // (H // G)
        heads.append(pooled_attention(q[:, i], k[:, g], v[:, g], m["scale"], m["mask"]["size"], m["mask"]["pool"]))
    return torch.cat(heads, -1) @ W[pre + "o"].T


# ------------------------------------------------------------------ generalised delta rule
def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(r, k, v, w, a, state=None):
    """r, k, v, w, a [T, H, D]; state [H, D, D] (key channel, value channel).  Both terms of a step read the
    old state.  Returns (o [T, H, D], state)."""
    T, H, D = r.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=r.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[-1], dtype=r.dtype)
    for t in range(T):
        for h in range(H):
            u = unit(k[t, h])
            old = S[h]
            S[h] = w[t, h][:, None] * old - torch.outer(a[t, h] * u, u @ old) + torch.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ r[t, h]
    return out, S


def decay_of(low, w2, w0):
    """Decay per channel from the low-rank projection (before its tanh)."""
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(torch.tanh(low) @ w2.T + w0))


def delta_mixer(h, m, W, pre, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    part = lambda x: x.reshape(T, H, D)  # noqa: E731
    r, k, v = (part(h @ W[pre + n].T) for n in ("r", "k", "v"))
    w = part(decay_of(h @ W[pre + "w1"].T, W[pre + "w2"], W[pre + "w0"]))
    a = part(torch.sigmoid(h @ W[pre + "a"].T + W[pre + "a.b"]))
    o, _ = delta_scan(r, k, v, w, a)
    y = rms_normalise(o, eps).reshape(T, H * D) * W[pre + "norm"] * torch.sigmoid(h @ W[pre + "g"].T)
    return y @ W[pre + "o"].T


def parallel_mixer(h, m, W, pre, eps):
    return (m["left_scale"] * attention_mixer(h, m["left"], W, pre + "left.", eps)
            + m["right_scale"] * delta_mixer(h, m["right"], W, pre + "right.", eps))


# ------------------------------------------------------------------ mixture of experts
def clamped_glu(gate, up, limit):
    g = torch.clamp(gate, max=limit)
    u = torch.clamp(up, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def expert(h, W, pre, limit):
    return clamped_glu(h @ W[pre + "gate"].T, h @ W[pre + "up"].T, limit) @ W[pre + "down"].T


def route(z, top, groups, scale):
    """z [E] router logits of one token -> {expert: weight}."""
    s = torch.sigmoid(z)
    E = s.numel()
    count, keep = (groups["count"], groups["keep"]) if groups else (1, 1)
    per = E // count
    score = [sum(sorted((float(x) for x in s[g * per:(g + 1) * per]), reverse=True)[:2]) for g in range(count)]
    best = sorted(range(count), key=lambda g: -score[g])[:keep]
    allowed = [e for e in range(E) if e // per in best]
    chosen = sorted(allowed, key=lambda e: -float(s[e]))[:top]
    total = sum(s[e] for e in chosen) + 1e-20
    return {e: s[e] / total * scale for e in chosen}


def moe(h, m, W, pre):
    r, T = m["router"], h.shape[0]
    out = torch.zeros_like(h)
    z = h @ W[pre + "router"].T
    every = [expert(h, W, f"{pre}e{e}.", m["expert"]["limit"]) for e in range(r["experts"])]
    for t in range(T):
        for e, w in route(z[t], r["top"], r.get("groups"), r["scale"]).items():
            out[t] += w * every[e][t]
    if m.get("shared"):
        out = out + torch.sigmoid(h @ W[pre + "shared.sg"].T) * expert(h, W, pre + "shared.", m["shared"]["limit"])
    return out


# ------------------------------------------------------------------ the whole model
def forward(cfg, W, tokens, layer_out=None):
    """tokens: list of ids of one sequence -> logits [T, vocab].  layer_out: a list that receives the
    residual after every layer."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{layer.get('weights_of', i)}."
        y = parallel_mixer(grouped_norm(x, W[p + "norm1"], eps, groups), layer["mixer"], W, p + "mix.", eps)
        if layer["mlp"] is not None:
            y = y + moe(grouped_norm(x, W[p + "norm2"], eps, groups), layer["mlp"], W, p + "mlp.")
        x = x + y
        if layer_out is not None:
            layer_out.append(x)
    return grouped_norm(x, W["final.norm"], eps, groups) @ W["embed"].T * cfg["logit_scale"]
