"""Each mechanism of the Golitar design alone, against the plain implementation in golitar_oracle.py:
on the CPU (the package's reference operations) and on the GPU (the HIP kernels, fp32 and bf16)."""

import math

import pytest
import torch

import golitar_oracle as O
from golitar_cases import rel_err
from neuronx_distributed_llama3_2_amd import ops
from neuronx_distributed_llama3_2_amd.modules.hybrid import interleaved_rope_tables

GPU = pytest.mark.gpu
# (device, activation type, relative tolerance)
WHERE = [pytest.param(("cpu", torch.float32, 2e-5), id="cpu"),
         pytest.param(("cuda", torch.float32, 5e-5), id="gpu-fp32", marks=GPU),
         pytest.param(("cuda", torch.bfloat16, 2e-2), id="gpu-bf16", marks=GPU)]


def rnd(*shape, seed=0, std=1.0, mean=0.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * std + mean


def act(t, where):   # rounded to the activation type; the oracle gets the rounded values too
    r = t.to(where[1])
    return r.to(where[0]), r.double()


def f32(t, where):
    return t.float().to(where[0])


# ------------------------------------------------------------------ hyper-connections
@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("S,W", [(1, 64), (2, 37), (4, 256), (8, 20)])
def test_hyper_step(where, S, W):
    M, eps = 5, 1e-5
    mix, wr, rd, nw, bias = rnd(S, S, seed=1), rnd(S, seed=2), rnd(S, seed=3), rnd(W, seed=4, std=0.3), rnd(W, seed=5)
    mix, wr, rd, nw, bias = (t.float().double() for t in (mix, wr, rd, nw, bias))
    embed, embed_o = act(rnd(11, W, seed=6), where)
    y, y_o = act(rnd(M, W, seed=7), where)
    ids = torch.tensor([3, 0, 10, 3, 7])
    streams = torch.full((M, S, W), 9.0, dtype=torch.float32, device=where[0])   # old contents do not matter
    h = ops.hyper_step(streams, read=f32(rd, where), norm_w=f32(nw, where), eps=eps, embed=embed, ids=ids.to(where[0]))
    x = embed_o[ids].unsqueeze(0).repeat(S, 1, 1)   # [S, M, W]
    assert rel_err(h, O.zero_centred_norm(O.hyper_read(x, rd), nw, eps)) < where[2]
    h = ops.hyper_step(streams, y=y, y_bias=f32(bias, where), mix=f32(mix, where), write=f32(wr, where),
                       read=f32(rd, where), norm_w=f32(nw, where), eps=eps)
    x = O.hyper_write(x, mix, wr, y_o + bias)
    assert rel_err(streams.transpose(0, 1), x) < 2e-5
    assert rel_err(h, O.zero_centred_norm(O.hyper_read(x, rd), nw, eps)) < where[2]
    # selected rows, read only: the model's last step
    rows = torch.tensor([4, 1])
    before = streams.clone()
    h = ops.hyper_step(streams, y=y, mix=f32(mix, where), write=f32(wr, where), read=torch.ones(S, device=where[0]),
                       norm_w=f32(nw, where), eps=eps, rows=rows.to(where[0]), store=False)
    want = O.zero_centred_norm(O.hyper_write(x, mix, wr, y_o).sum(0), nw, eps)[rows]
    assert rel_err(h, want) < where[2]
    assert torch.equal(streams, before)


@pytest.mark.parametrize("where", WHERE)
def test_squared_relu_and_softcap(where):
    x, xo = act(rnd(3, 41), where)
    assert rel_err(ops.relu_squared(x), torch.clamp(xo, min=0) ** 2) < where[2]
    z = f32(rnd(7, 13, std=20.0), where)
    zo = z.double().cpu()
    assert rel_err(ops.softcap_(z, 7.5), 7.5 * torch.tanh(zo / 7.5)) < 2e-5


# ------------------------------------------------------------------ gated delta rule
def delta_case(where, B, T, H, G, D, V, taps, seed=0, strong=False):
    sz = ops.DeltaSizes(H, G, D, V)
    n = (sz.columns + 15) // 16 * 16
    proj, proj_o = act(rnd(B, T, n, seed=seed), where)
    conv = rnd(taps, sz.channels, seed=seed + 1, std=0.6).float()
    # strong: most heads forget within a token or two, so sums of log decays grow large
    a_log = rnd(H, seed=seed + 2, std=0.5, mean=3.0 if strong else -1.0).float()
    dt = rnd(H, seed=seed + 3, std=0.5, mean=-1.0).float()
    norm = rnd(V, seed=seed + 4, std=0.2, mean=1.0).float()
    return sz, proj, proj_o, conv, a_log, dt, norm


def delta_oracle(sz, proj, conv, a_log, dt, norm, eps):
    """proj [T, columns] of one sequence -> [T, H V]."""
    H, G, D, V, C = sz.heads, sz.kv_heads, sz.dim, sz.vdim, sz.channels
    T = proj.shape[0]
    x = O.silu(O.causal_conv(proj[:, :C], conv.double().t()))
    rep = [h // (H // G) for h in range(H)]
    q = (O.unit(x[:, :G * D].view(T, G, D)) * D ** -0.5)[:, rep]
    k = O.unit(x[:, G * D:2 * G * D].view(T, G, D))[:, rep]
    gates = proj[:, C + H * V:]
    beta = torch.sigmoid(gates[:, :H])
    decay = torch.exp(-torch.exp(a_log.double()) * O.softplus(gates[:, H:2 * H] + dt.double()))
    o, _ = O.delta_scan(q, k, x[:, 2 * G * D:C].reshape(T, H, V), decay, beta)
    o = O.rms_normalise(o, eps) * norm.double() * O.silu(proj[:, C:C + H * V]).view(T, H, V)
    return o.reshape(T, H * V)


def run_delta(where, case, cuts, lengths, slots, state, ring, chunk_from, fused=True, eps=1e-5):
    sz, proj, _, conv, a_log, dt, norm = case
    B, T, n = proj.shape
    d = where[0]
    outs, t0 = [], 0
    for c in cuts:
        left = (torch.tensor(lengths) - t0).clamp(0, c).to(torch.int32)
        full = bool((left == c).all())
        y = ops.delta_rule(proj[:, t0:t0 + c].reshape(B * c, n).contiguous(), B, c, sz, conv.to(d), a_log.to(d), dt.to(d),
                           norm.to(d), eps, torch.full((B,), t0, dtype=torch.long, device=d),
                           None if full else left.to(d), slots.to(d), state, ring, fused, chunk_from)
        outs.append(y.view(B, c, -1))
        t0 += c
    return torch.cat(outs, 1)


SIZES = [(1, 1, 8, 8, 1), (4, 2, 24, 40, 4), (3, 3, 33, 20, 2), (2, 1, 128, 96, 4), (2, 2, 72, 130, 6)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,V,taps", SIZES)
def test_delta_rule(where, H, G, D, V, taps):
    """Two sequences of different lengths, whole (in chunks and token by token), in portions of several
    sizes and decoded one by one; slots that held something else before."""
    B, T, lens = 2, 75, [75, 41]
    case = delta_case(where, B, T, H, G, D, V, taps)
    sz, proj, proj_o = case[:3]
    want = [delta_oracle(sz, proj_o[b, :lens[b]], *case[3:], 1e-5) for b in range(B)]
    slots = torch.tensor([2, 0], dtype=torch.int32)
    plans = [([75], 32), ([75], 1000), ([2, 64, 1, 1, 7], 32), ([33, 2, 40], 2)]
    if where[0] == "cpu":
        plans = [plans[0], plans[2]]
    for cuts, chunk_from in plans:
        state = torch.full((3, H, V, sz.padded_dim), 5.0, device=where[0])
        state[..., D:] = 0
        ring = torch.full((3, taps, sz.channels), -3.0, dtype=where[1], device=where[0])
        got = run_delta(where, case, cuts, lens, slots, state, ring, chunk_from)
        for b in range(B):
            assert rel_err(got[b, :lens[b]], want[b]) < where[2], (cuts, chunk_from, b)
            assert torch.isfinite(got[b].float()).all()
        assert bool((state[1, ..., :D] == 5.0).all()) and bool((ring[1] == -3.0).all())   # another's slot


@pytest.mark.parametrize("where", WHERE)
def test_delta_rule_strong_decay(where):
    """Sums of log decays in the hundreds: their differences must not lose the small ones."""
    case = delta_case(where, 1, 140, 2, 2, 32, 16, 3, seed=9, strong=True)
    sz, proj, proj_o = case[:3]
    want = delta_oracle(sz, proj_o[0], *case[3:], 1e-5)
    state = torch.zeros((1, 2, 16, 32), device=where[0])
    ring = torch.zeros((1, 3, sz.channels), dtype=where[1], device=where[0])
    got = run_delta(where, case, [140], [140], torch.zeros(1, dtype=torch.int32), state, ring, 32)
    assert rel_err(got[0], want) < where[2]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("cuts", [[1] * 12, [5] + [1] * 7, [70] + [1] * 5])
def test_delta_rule_decode(where, cuts):
    """The one-token launch against the several-token ones, from the first token on."""
    T = sum(cuts)
    case = delta_case(where, 2, T, 4, 2, 24, 72, 4, seed=3)
    sz, proj, proj_o = case[:3]
    for fused in (True, False):
        state = torch.full((2, 4, 72, 32), 2.0, device=where[0])
        state[..., 24:] = 0
        ring = torch.full((2, 4, sz.channels), 2.0, dtype=where[1], device=where[0])
        got = run_delta(where, case, cuts, [T, T], torch.tensor([1, 0], dtype=torch.int32), state, ring, 32, fused)
        for b in range(2):
            assert rel_err(got[b], delta_oracle(sz, proj_o[b], *case[3:], 1e-5)) < where[2]


def test_delta_rule_reads_out_after_the_write():
    """What the read-out order changes is visible: reading before the write differs from the oracle."""
    q = O.unit(rnd(3, 1, 4))
    v, one = rnd(3, 1, 5, seed=2), torch.ones(3, 1, dtype=torch.float64)
    o, _ = O.delta_scan(q, q, v, one, one)
    assert torch.allclose(o, v, atol=1e-5)   # beta = 1: a key's read-out is what was just written under it


# ------------------------------------------------------------------ differential attention
def rope(rot_dims, max_pos, base=10000.0, scaling=True):
    sc = dict(factor=8.0, low=1.0, high=4.0, original=64.0) if scaling else {}
    cos, sin = interleaved_rope_tables(rot_dims, base, max_pos, **sc)
    return cos, sin, O.rotary_frequencies({"dims": rot_dims, "base": base, "scaling": sc or None})


@pytest.mark.parametrize("dims,base,scaling", [(8, 10000.0, True), (24, 500000.0, True), (6, 100.0, False), (0, 10.0, True)])
def test_rotary_tables(dims, base, scaling):
    cos, sin, freqs = rope(dims, 300, base, scaling)
    assert cos.shape == (300, dims // 2)
    for p in (0, 1, 77, 299):
        for i, f in enumerate(freqs):
            assert abs(float(cos[p, i]) - math.cos(p * f)) < 1e-6 and abs(float(sin[p, i]) - math.sin(p * f)) < 1e-6
    if scaling and dims == 24:   # all three bands occur
        plain = O.rotary_frequencies({"dims": dims, "base": base, "scaling": None})
        ratio = [a / b for a, b in zip(freqs, plain)]
        assert ratio[0] == 1.0 and abs(ratio[-1] - 1 / 8) < 1e-12 and any(1 / 8 + 1e-3 < r < 1 - 1e-3 for r in ratio)


class Attn:
    """One attention layer's inputs for B sequences of T tokens, and the oracle on them."""

    def __init__(self, where, B, T, H, G, R, D, V, rot, window, softcap, cap, scale=0.3, seed=0, amp=1.0):
        self.where, self.B, self.T, self.window = where, B, T, window
        self.sz = ops.AttnSizes(H, G, R, D, V)
        self.n = (self.sz.columns + 15) // 16 * 16
        self.buf, self.buf_o = act(rnd(B, T, self.n, seed=seed) * amp, where)
        self.bias = rnd(self.sz.columns, seed=seed + 1, std=0.3).float()
        self.qn, self.kn = rnd(D, seed=seed + 2, std=0.3, mean=1.2).float(), rnd(D, seed=seed + 3, std=0.3, mean=1.2).float()
        self.cos, self.sin, self.freqs = rope(rot, 4096)
        self.rule = ops.AttnRule(scale, softcap, window, 0.37 if R == 2 else 0.0, 0.6 if R == 2 else 1.0, 1e-6)
        self.cap = cap
        z = lambda *s: torch.full(s, 7.0, dtype=where[1], device=where[0])  # noqa: E731  (stale contents)
        self.kc, self.vc = z(B + 1, G * R, cap, D), z(B + 1, G, cap, V)
        self.slots = torch.arange(B, 0, -1, dtype=torch.int32, device=where[0])
        self.tickets = torch.zeros((B + 1) * H, dtype=torch.int32, device=where[0])

    def step(self, t0, n, prompt, lengths=None, fused=True, decode=False):
        d, B = self.where[0], self.B
        to = lambda t: t.to(d)  # noqa: E731
        buf = self.buf[:, t0:t0 + n].reshape(B * n, self.n).clone()
        pos = torch.full((B, 1), t0, dtype=torch.long, device=d)
        lens = torch.tensor(lengths, dtype=torch.int32, device=d) if lengths is not None else None
        prep = (to(self.bias), to(self.qn), to(self.kn), 1e-5, to(self.cos), to(self.sin), pos)
        if decode:
            y = ops.attn_decode(buf, self.sz, self.rule, *prep, self.slots, self.kc, self.vc, self.tickets)
            assert int(self.tickets.abs().sum()) == 0
        else:
            ops.attn_prep_(buf, B, n, self.sz, *prep, lens, self.slots, self.kc, self.vc)
            y = ops.window_attention(buf, B, n, self.sz, self.rule, pos, lens, self.slots, self.kc, self.vc, prompt, fused)
        return y.view(B, n, -1)

    def oracle(self, b, T, window="own"):
        window = (self.window or None) if window == "own" else window
        sz = self.sz
        x = self.buf_o[b, :T, :sz.columns] + self.bias.double()
        q = x[:, :sz.q_columns].reshape(T, sz.heads, sz.maps, sz.dim)
        k = x[:, sz.q_columns:sz.q_columns + sz.k_columns].reshape(T, sz.kv_heads, sz.maps, sz.dim)
        v = x[:, sz.q_columns + sz.k_columns:].reshape(T, sz.kv_heads, sz.vdim)
        q = O.rotate_interleaved(O.rms_normalise(q, 1e-5) * self.qn.double(), self.freqs)
        k = O.rotate_interleaved(O.rms_normalise(k, 1e-5) * self.kn.double(), self.freqs)
        heads = []
        for h in range(sz.heads):
            g = h // (sz.heads // sz.kv_heads)
            a = [O.attention_map(q[:, h, c], k[:, g, c], v[:, g], self.rule.scale, self.rule.softcap or None, window)
                 for c in range(sz.maps)]
            o = a[0]
            if sz.maps == 2:
                o = O.rms_normalise(a[0] - self.rule.lam * a[1], self.rule.eps) * self.rule.out_scale
            heads.append(o)
        return torch.cat(heads, -1)


ATTN = [  # H, G, maps, D, V, rot, window, softcap
    (4, 2, 2, 16, 24, 8, 37, 20.0), (2, 1, 2, 40, 64, 40, 64, 30.0), (3, 3, 2, 10, 6, 2, 1, 60.0),
    (2, 2, 2, 72, 136, 64, 90, 50.0), (2, 1, 1, 48, 32, 16, 0, 0.0), (2, 1, 2, 64, 128, 0, 0, 30.0), (1, 1, 2, 128, 256, 2, 5, 0.0),
    (8, 2, 2, 24, 40, 12, 70, 30.0), (4, 1, 1, 104, 72, 8, 0, 25.0), (12, 3, 2, 40, 160, 0, 100, 0.0)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,R,D,V,rot,window,softcap", ATTN)
def test_attention(where, H, G, R, D, V, rot, window, softcap):
    """Prompts (matrix-core and row kernels) of unequal lengths, then portions, then decoding over a ring
    that wraps, against the oracle."""
    B, T = 2, 170
    a = Attn(where, B, T, H, G, R, D, V, rot, window, softcap, cap=min(window + 15 if window else T, T))
    want = [a.oracle(b, T) for b in range(B)]
    tol = where[2] if where[1] != torch.bfloat16 else 4e-2   # bf16: q and k are rounded after their norms
    for fused in (False, True) if where[0] == "cuda" else (True,):
        lens = [140, 97]
        got = a.step(0, 140, True, lens, fused=fused)
        for b in range(B):
            assert rel_err(got[b, :lens[b]], want[b][:lens[b]]) < tol, fused
        got = a.step(0, 140, True, None, fused=fused)
        t = 140
        for n in (2, 7, 15):
            got = a.step(t, n, False, None, fused=fused)
            for b in range(B):
                assert rel_err(got[b], want[b][t:t + n]) < tol, (fused, n)
            t += n
        for decode in (True, False, True, True):
            got = a.step(t, 1, False, None, fused=fused, decode=decode)
            for b in range(B):
                assert rel_err(got[b], want[b][t:t + 1]) < tol, (fused, "decode", decode)
            t += 1
        assert bool((a.kc[0] == 7.0).all()) and bool((a.vc[0] == 7.0).all())   # nobody's slot


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("window", [1, 2, 63, 64, 65, 130])
def test_window_edges(where, window):
    """A key that outweighs all others just inside or just outside the window, in a prompt and in decoding:
    one token more or less of window changes the output completely."""
    T, D = 200, 16
    cap = min(window + 15, T)
    for age in (window - 1, window):   # the last key seen, the first one not seen
        a = Attn(where, 1, T, 1, 1, 2, D, 8, 0, window, 20.0, cap, scale=1.0, seed=5)
        a.bias.zero_()
        for i in (0, 63, 64, 127, 128, 150):   # queries; each finds its key `age` tokens back
            if i - age < 0:
                continue
            for c in range(2):   # a strong match in both maps, of different values
                probe = rnd(D, seed=50 + c)
                a.buf_o[0, i, c * D:(c + 1) * D] = probe
                a.buf_o[0, i - age, 2 * D + c * D:2 * D + (c + 1) * D] = probe * (1 if c == 0 else -1)
        a.buf = a.buf_o.to(where[1]).to(where[0])
        a.buf_o = a.buf.double().cpu()
        want, wrong = a.oracle(0, T), a.oracle(0, T, window + 1)
        tol = where[2] if where[1] != torch.bfloat16 else 4e-2
        got = a.step(0, T, True)[0].double().cpu()
        assert rel_err(got, want) < tol
        if age == window:
            assert rel_err(wrong, want) > 0.2   # the oracle with one token more is far off
        a.step(0, 100, True)
        for t in range(100, 152):
            assert rel_err(a.step(t, 1, False, decode=t % 3 != 0)[0], want[t:t + 1]) < tol, t


@pytest.mark.parametrize("where", WHERE)
def test_first_tokens_see_only_what_is_there(where):
    """Sequences of one and two tokens, prompt and decode, over a cache full of another sequence's keys."""
    a = Attn(where, 2, 4, 4, 2, 2, 16, 24, 8, 37, 20.0, cap=52)
    want = [a.oracle(b, 4) for b in range(2)]
    tol = where[2] if where[1] != torch.bfloat16 else 4e-2
    for first in (1, 2):
        got = a.step(0, first, True)
        for b in range(2):
            assert rel_err(got[b], want[b][:first]) < tol
        for t in range(first, 4):
            got = a.step(t, 1, False, decode=True)
            for b in range(2):
                assert rel_err(got[b], want[b][t:t + 1]) < tol


@pytest.mark.gpu
@pytest.mark.parametrize("visible", [63, 64, 65, 255, 257, 600, 2200])
@pytest.mark.parametrize("heads,vdim", [(2, 12), (4, 24)])   # any-size kernel; four heads a workgroup
def test_split_decode(visible, heads, vdim):
    """Decoding over many visible keys (several workgroups per head and a merge), repeated: the
    arrival counters are left at zero; a key that outweighs all others is far away."""
    where = ("cuda", torch.float32, 5e-5)
    T = visible + 40
    a = Attn(where, 1, T, heads, 1, 2, 16, vdim, 0, visible, 20.0, cap=visible + 15, scale=1.0, seed=8)
    a.bias.zero_()
    probe = rnd(16, seed=60)
    k0 = heads * 32   # the first key column
    for i in range(T - 3, T):
        a.buf_o[0, i, :16] = probe
        a.buf_o[0, i - visible + 1, k0:k0 + 16] = probe * 1.5
    a.buf = a.buf_o.to(where[1]).to(where[0])
    a.buf_o = a.buf.double().cpu()
    want = a.oracle(0, T)
    a.step(0, T - 3, True)
    for t in range(T - 3, T):
        assert rel_err(a.step(t, 1, False, decode=True)[0], want[t:t + 1]) < where[2]


@pytest.mark.gpu
@pytest.mark.parametrize("B,H,G", [(16, 8, 2), (40, 8, 2), (48, 6, 3)])
def test_decode_shares_keys_between_heads(B, H, G):
    """Enough sequences that several query heads of a key / value head share a workgroup, against the
    one-wave-a-query kernel on the same cache; some sequences are much shorter than the window."""
    where = ("cuda", torch.float32, 5e-5)
    a = Attn(where, B, 150, H, G, 2, 24, 40, 8, 130, 20.0, cap=150, seed=12)
    a.step(0, 149, True)
    pos = torch.randint(0, 150, (B, 1), generator=torch.Generator().manual_seed(3)).cuda()
    buf = a.buf[:, 149].contiguous()
    prep = (a.bias.cuda(), a.qn.cuda(), a.kn.cuda(), 1e-5, a.cos.cuda(), a.sin.cuda(), pos)
    kc, vc = a.kc.clone(), a.vc.clone()
    got = ops.attn_decode(buf, a.sz, a.rule, *prep, a.slots, kc, vc, a.tickets)
    row = buf.clone()
    ops.attn_prep_(row, B, 1, a.sz, *prep, None, a.slots, a.kc, a.vc)
    want = ops.window_attention(row, B, 1, a.sz, a.rule, pos, None, a.slots, a.kc, a.vc, False, False)
    assert rel_err(got, want.cpu()) < 5e-5
    assert rel_err(kc.flatten(0, 2), a.kc.flatten(0, 2).cpu()) < 1e-5 and torch.equal(vc, a.vc)
    assert int(a.tickets.abs().sum()) == 0


# ------------------------------------------------------------------ fused decode projections
@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 2, 3, 4])
@pytest.mark.parametrize("N,K", [(80, 72), (33, 8), (200, 2048), (1000, 1000), (48, 4096), (24, 6144)])
def test_decode_projections(M, N, K):
    d, bf = "cuda", torch.bfloat16
    w = (rnd(N, K) * K ** -0.5).to(bf)
    x, u, nw = rnd(M, K, seed=1).to(bf), rnd(M, K, seed=2, std=3.0).float(), rnd(K, seed=3, std=0.2).float()
    wd, wo = w.to(d), w.double()
    assert rel_err(ops.decode_linear(wd, x.to(d)), x.double() @ wo.T) < 5e-3
    h = O.zero_centred_norm(u.double(), nw.double(), 1e-5).to(bf).double() @ wo.T
    norm = (None, u.to(d), nw.to(d), 1e-5)
    assert rel_err(ops.decode_linear(wd, *norm), h) < 8e-3
    assert rel_err(ops.decode_linear(wd, *norm, "relu2"), torch.clamp(h, min=0) ** 2) < 1.6e-2
    assert rel_err(ops.decode_linear(wd, *norm, "f32", 2.5), 2.5 * torch.tanh(h / 2.5)) < 5e-3
    for S in (1, 3, 8):
        st, mix, wr, rd, b = rnd(M, S, N), rnd(S, S, seed=4), rnd(S, seed=5), rnd(S, seed=6), rnd(N, seed=7)
        f = lambda t: t.float().to(d)  # noqa: E731
        streams = f(st)
        un = ops.decode_linear_into_streams(wd, x.to(d), streams, f(b), f(mix), f(wr), f(rd))
        new = O.hyper_write(st.transpose(0, 1), mix, wr, x.double() @ wo.T + b)
        assert rel_err(streams.transpose(0, 1).reshape(S * M, N), new.reshape(S * M, N)) < 1e-2
        assert rel_err(un, O.hyper_read(new, rd)) < 2e-2
