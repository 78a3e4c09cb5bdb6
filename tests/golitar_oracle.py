"""Plain, slow implementation of the Golitar design, one function per mechanism (the tests' oracle).

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


def zero_centred_norm(x, w, eps):
    return rms_normalise(x, eps) * (1 + w)


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


# ------------------------------------------------------------------ hyper-connections
def hyper_read(streams, w_in):
    """streams [S, T, W] -> the sublayer's input [T, W]."""
    return sum(w_in[s] * streams[s] for s in range(streams.shape[0]))


def hyper_write(streams, mix, w_out, y):
    """new_t = sum_s mix[s, t] old_s + out[t] y."""
    S = streams.shape[0]
    return torch.stack([sum(mix[s, t] * streams[s] for s in range(S)) + w_out[t] * y for t in range(S)])


# ------------------------------------------------------------------ gated delta rule
def causal_conv(x, taps):
    """x [T, C], taps [C, n] (last column = current token) -> [T, C]; zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for j in range(n):
        back = n - 1 - j   # column j meets the input `back` tokens ago
        if back < T:
            out[back:] += taps[:, j] * x[:T - back]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, decay, beta, state=None):
    """q, k [T, H, D] v [T, H, V] decay, beta [T, H]; returns (o [T, H, V], state [H, D, V])."""
    T, H, D = q.shape
    V = v.shape[-1]
    S = torch.zeros(H, D, V, dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, V, dtype=q.dtype)
    for t in range(T):
        S = S * decay[t][:, None, None]
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + torch.einsum("hd,hv->hdv", k[t], u)
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out, S


def delta_mixer(h, m, W, pre, eps):
    """h [T, width] -> [T, width]; m = the layer's mixer sizes, W the weights, pre 'l<i>.mix.'."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    mixed = {}
    for n in ("q", "k", "v"):
        mixed[n] = silu(causal_conv(h @ W[pre + n].T, W[pre + n + ".conv"]))
    q = unit(mixed["q"].view(T, G, D)) * D ** -0.5
    k = unit(mixed["k"].view(T, G, D))
    head_of = [i // (H // G) for i in range(H)]
    q, k = q[:, head_of], k[:, head_of]
    beta = torch.sigmoid(h @ W[pre + "b"].T)
    decay = torch.exp(-torch.exp(W[pre + "A_log"]) * softplus(h @ W[pre + "a"].T + W[pre + "dt_bias"]))
    o, _ = delta_scan(q, k, mixed["v"].view(T, H, V), decay, beta)
    o = rms_normalise(o, eps) * W[pre + "norm"] * silu(h @ W[pre + "g"].T).view(T, H, V)
    return o.reshape(T, H * V) @ W[pre + "o"].T


# ------------------------------------------------------------------ differential attention
def rotary_frequencies(rot):
    n = rot["dims"]
    f = [float(rot["base"]) ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if sc:
        out = []
        for x in f:
            l = 2 * math.pi / x
            if l < sc["original"] / sc["high"]:
                out.append(x)
            elif l > sc["original"] / sc["low"]:
                out.append(x / sc["factor"])
            else:
                s = (sc["original"] / l - sc["low"]) / (sc["high"] - sc["low"])
                out.append((1 - s) * x / sc["factor"] + s * x)
        f = out
    return f


def rotate_interleaved(x, freqs, pos0=0):
    """x [T, ..., D]: pair (2i, 2i + 1) of row t turned by (pos0 + t) freqs[i]; the rest unchanged."""
    out = x.clone()
    pos = torch.arange(pos0, pos0 + x.shape[0], dtype=x.dtype).view((-1,) + (1,) * (x.dim() - 2))
    for i, f in enumerate(freqs):
        c, s = torch.cos(pos * f), torch.sin(pos * f)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def visible(i, j, window):
    return j <= i and (window is None or i - j < window)


def attention_map(q, k, v, scale, softcap, window):
    """One head's map: q, k [T, D], v [T, V] -> [T, V]."""
    T = q.shape[0]
    seen = torch.tensor([[visible(i, j, window) for j in range(T)] for i in range(T)])
    s = (q @ k.T) * scale
    if softcap:
        s = softcap * torch.tanh(s / softcap)
    return torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v


def lambda_of(W, pre, diff):
    e = lambda a, b: torch.exp((W[pre + a] * W[pre + b]).sum())  # noqa: E731
    return e("lq1", "lk1") - e("lq2", "lk2") + diff


def differential_attention(h, m, W, pre, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ W[pre + "q"].T + W[pre + "q.b"]).view(T, H, 2, D)
    k = (h @ W[pre + "k"].T + W[pre + "k.b"]).view(T, G, 2, D)
    v = (h @ W[pre + "v"].T + W[pre + "v.b"]).view(T, G, V)
    q = rms_normalise(q, eps) * W[pre + "q.norm"]
    k = rms_normalise(k, eps) * W[pre + "k.norm"]
    f = rotary_frequencies(m["rot"])
    q, k = rotate_interleaved(q, f), rotate_interleaved(k, f)
    lam = lambda_of(W, pre, m["diff"])
    window = m["mask"]["size"] if m.get("mask") else None
    heads = []
    for i in range(H):
        g = i // (H // G)
        a = [attention_map(q[:, i, c], k[:, g, c], v[:, g], m["scale"], m.get("softcap"), window) for c in range(2)]
        heads.append(rms_normalise(a[0] - lam * a[1], eps) * (1 - m["diff"]))
    return torch.cat(heads, -1) @ W[pre + "o"].T + W[pre + "o.b"]


# ------------------------------------------------------------------ feed-forward and the whole model
def relu_squared_mlp(h, W, pre):
    return torch.clamp(h @ W[pre + "up"].T, min=0) ** 2 @ W[pre + "down"].T


def forward(cfg, W, tokens, layer_out=None):
    """tokens: list of ids of one sequence -> logits [T, vocab].  layer_out: a list that receives the
    summed residual streams after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    streams = torch.stack([x] * cfg["streams"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        for q in (1, 2) if layer["mlp"] is not None else (1,):
            hc = f"{p}hc{q}."
            h = zero_centred_norm(hyper_read(streams, W[hc + "in"]), W[f"{p}norm{q}"], eps)
            if q == 2:
                y = relu_squared_mlp(h, W, p + "mlp.")
            elif layer["type"] == "delta":
                y = delta_mixer(h, layer["mixer"], W, p + "mix.", eps)
            else:
                y = differential_attention(h, layer["mixer"], W, p + "mix.", eps)
            streams = hyper_write(streams, W[hc + "mix"], W[hc + "out"], y)
        if layer_out is not None:
            layer_out.append(streams.sum(0))
    logits = zero_centred_norm(streams.sum(0), W["final.norm"], eps) @ W["head"].T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
