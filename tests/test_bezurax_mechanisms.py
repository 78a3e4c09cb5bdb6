"""Each mechanism of the Bezurax design alone, against the plain implementation in bezurax_oracle.py: on the
CPU (the package's reference operations) and on the GPU (the HIP kernels, fp32 and bf16)."""

import math

import pytest
import torch

import bezurax_oracle as O
from golitar_cases import rel_err
from neuronx_distributed_llama3_2_amd import ops
from neuronx_distributed_llama3_2_amd.modules.hybrid import ChannelDelta, ParallelMixer, PooledAttention, RoutedExperts, StepContext
from neuronx_distributed_llama3_2_amd.ops.pooled_attention import blocks_seen

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


# ------------------------------------------------------------------ residual sum and grouped norms
@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("W,groups", [(64, 1), (96, 3), (40, 8), (45, 5), (1300, 2), (2048, 16), (33, 33)])
def test_residual_norms(where, W, groups):
    M, eps = 5, 1e-5
    ws = [rnd(W, seed=1 + i, std=0.3, mean=1.0).float() for i in range(2)]
    embed, embed_o = act(rnd(11, W, seed=6) * torch.linspace(0.1, 6, W), where)   # parts of different size
    ids = torch.tensor([3, 0, 10, 3, 7])
    x = torch.full((M, W), 9.0, dtype=torch.float32, device=where[0])   # old contents do not matter
    norm = lambda v, i: O.grouped_norm(v, ws[i].double(), eps, groups)  # noqa: E731
    hs = ops.residual_norms(x, [f32(w, where) for w in ws], eps, groups, embed=embed, ids=ids.to(where[0]))
    ref = embed_o[ids]
    for i, h in enumerate(hs):
        assert rel_err(h, norm(ref, i)) < where[2]
    adds = [act(rnd(M, W, seed=7 + i), where) for i in range(2)]
    pairs, pairs_o = act(rnd(3 * M, W, seed=9), where)
    inverse = torch.randperm(3 * M, generator=torch.Generator().manual_seed(2)).view(M, 3).int()
    hs = ops.residual_norms(x, [f32(ws[1], where)], eps, groups, adds=[a for a, _ in adds], pairs=pairs,
                            inverse=inverse.to(where[0]))
    ref = ref + adds[0][1] + adds[1][1] + pairs_o[inverse.long()].sum(1)
    assert rel_err(x, ref) < 2e-5
    assert rel_err(hs[0], norm(ref, 1)) < where[2]
    if groups > 1:
        assert rel_err(O.grouped_norm(ref, ws[1].double(), eps, 1), norm(ref, 1)) > 0.02
    # chosen rows, read only: the model's last step
    rows, before = torch.tensor([4, 1]), x.clone()
    hs = ops.residual_norms(x, [f32(ws[0], where)], eps, groups, adds=[adds[0][0]], rows=rows.to(where[0]), store=False)
    assert rel_err(hs[0], norm(ref + adds[0][1], 0)[rows]) < where[2]
    assert torch.equal(x, before)


@pytest.mark.parametrize("where", WHERE)
def test_norm_of_small_rows_needs_eps_inside_the_root(where):
    x = f32(rnd(2, 12, std=1e-3), where)
    w = torch.ones(12)
    h = ops.residual_norms(x, [w.to(where[0])], 1e-5, 3, dtype=where[1])[0]
    assert rel_err(h, O.grouped_norm(x.double().cpu(), w.double(), 1e-5, 3)) < where[2]


# ------------------------------------------------------------------ router and experts
def router_cases():
    return [(6, 2, 3, 2, 1.7), (10, 4, 2, 1, 2.2), (4, 1, 4, 2, 1.0), (1, 1, 1, 1, 0.5), (5, 5, 1, 1, 1.0), (128, 8, 8, 4, 2.5),
            (96, 6, 1, 1, 1.0), (12, 4, 6, 3, 3.0)]


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("E,top,count,keep,scale", router_cases())
@pytest.mark.parametrize("M", [1, 3, 77])
def test_router(where, E, top, count, keep, scale, M):
    logits = f32(rnd(M, E + 3, seed=E, std=1.5), where)
    rule = ops.RouterRule(E, top, scale, count, keep)
    r = ops.route(logits[:, :E], rule)   # (rows with a stride)
    offs, token, weight, inverse = (t.cpu() for t in (r.offs, r.token, r.weight, r.inverse))
    assert offs[0] == 0 and offs[-1] == M * top
    assert sorted(inverse.reshape(-1).tolist()) == list(range(M * top))
    for m in range(M):
        want = O.route(logits[m, :E].double().cpu(), top, {"count": count, "keep": keep}, scale)
        got = {}
        for row in inverse[m].tolist():
            assert int(token[row]) == m
            e = int((offs[1:] <= row).sum())
            got[e] = float(weight[row])
        assert set(got) == set(want)
        for e, w in want.items():
            assert abs(got[e] - float(w)) < 1e-5 * scale


@pytest.mark.parametrize("where", WHERE[:2])
def test_router_keeps_to_the_best_groups(where):
    """The largest score of all is in a group whose two best sum to less: it is not chosen."""
    z = torch.tensor([[9.0, -9.0, -9.0, 2.0, 2.0, -9.0, 1.0, -9.0, 0.5]], device=where[0])
    r = ops.route(z, ops.RouterRule(9, 2, 1.0, 3, 1))
    chosen = lambda r: {int((r.offs.cpu()[1:] <= i).sum()) for i in r.inverse.cpu()[0].tolist()}  # noqa: E731
    assert chosen(r) == {3, 4}
    assert 0 in chosen(ops.route(z, ops.RouterRule(9, 2, 1.0, 3, 3)))


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("F", [8, 17, 64])
def test_clamped_activation(where, F):
    gu, gu_o = act(rnd(9, 2 * F, std=2.0), where)
    weight, gate = f32(rnd(9, seed=1), where), f32(rnd(9, 5, seed=2), where)
    want = O.clamped_glu(gu_o[:, :F], gu_o[:, F:], 0.9)
    assert rel_err(ops.clamped_glu(gu, 0.9), want) < where[2]
    assert rel_err(ops.clamped_glu(gu, 0.9, weight), want * weight.double().cpu()[:, None]) < where[2]
    assert rel_err(ops.clamped_glu(gu, 0.9, gate[:, 3], sigmoid=True), want * torch.sigmoid(gate[:, 3].double().cpu())[:, None]) < where[2]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("E,N,K", [(5, 24, 40), (3, 17, 9), (4, 136, 64), (7, 64, 256)])
@pytest.mark.parametrize("M", [2, 60, 2500])
def test_expert_products(where, E, N, K, M):
    w, w_o = act(rnd(E, N, K) * K ** -0.5, where)
    x, x_o = act(rnd(M, K, seed=1), where)
    top = 2
    r = ops.route(f32(rnd(M, E, seed=2, std=2.0), where), ops.RouterRule(E, top))
    offs, token = r.offs.cpu(), r.token.cpu().long()
    want = torch.empty(M * top, N, dtype=torch.float64)
    for e in range(E):
        want[offs[e]:offs[e + 1]] = x_o[token[offs[e]:offs[e + 1]]] @ w_o[e].T
    y = ops.expert_linear_rows(x, w, r.offs, r.token)
    assert rel_err(y, want) < where[2]
    x2, x2_o = act(x_o[token], where)
    assert rel_err(ops.expert_linear_rows(x2, w, r.offs), want) < where[2]


def experts_module(where, W, E, top, ff, limit, scale, groups, keep, shared_ff, shared_limit, seed=0):
    dt, dev = where[1], where[0]
    mod = RoutedExperts(W, ops.RouterRule(E, top, scale, groups, keep), ff, limit, shared_ff, shared_limit, dt, dev)
    sd = {"router": rnd(E, W, seed=seed + 1) * 2 * W ** -0.5, "shared.sg": rnd(1, W, seed=seed + 2) * W ** -0.5}
    for e in range(E):
        for i, (n, s) in enumerate((("gate", (ff, W)), ("up", (ff, W)), ("down", (W, ff)))):
            sd[f"e{e}.{n}"] = rnd(*s, seed=seed + 10 * e + i + 3) * s[1] ** -0.5
    for i, (n, s) in enumerate((("gate", (shared_ff, W)), ("up", (shared_ff, W)), ("down", (W, shared_ff)))):
        sd["shared." + n] = rnd(*s, seed=seed + 900 + i) * max(s[1], 1) ** -0.5
    sd = {k: v.to(dt).double() for k, v in sd.items()}
    mod.router.weight.data.zero_()
    mod.router.weight.data[:E] = sd["router"].to(dt)
    mod.gate_up.data.copy_(torch.stack([torch.cat([sd[f"e{e}.gate"], sd[f"e{e}.up"]]) for e in range(E)]))
    mod.down.data.copy_(torch.stack([sd[f"e{e}.down"] for e in range(E)]))
    cfg = {"router": {"experts": E, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}},
           "expert": {"ff": ff, "limit": limit}}
    if shared_ff:
        mod.router.weight.data[E] = sd["shared.sg"][0].to(dt)
        mod.shared_up.weight.data.copy_(torch.cat([sd["shared.gate"], sd["shared.up"]]))
        mod.shared_down.weight.data.copy_(sd["shared.down"])
        cfg["shared"] = {"ff": shared_ff, "limit": shared_limit}
    for p in mod.parameters():
        p.requires_grad_(False)
    return mod, cfg, sd


MOES = [(48, 6, 2, 24, 1.2, 1.7, 3, 2, 40, 0.8), (64, 10, 4, 32, 0.6, 2.2, 2, 1, 64, 1.1), (36, 5, 5, 17, 1.0, 1.0, 1, 1, 0, 0.0),
        (128, 16, 3, 64, 7.0, 1.0, 4, 2, 128, 7.0), (64, 1, 1, 8, 1.0, 0.5, 1, 1, 24, 0.3)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("case", MOES)
@pytest.mark.parametrize("M", [1, 4, 17, 33, 64, 90])
def test_routed_experts(where, case, M):
    """The whole feed-forward, as it reaches the residual, for a few tokens (unsorted kernels) and many."""
    mod, cfg, sd = experts_module(where, *case)
    W = case[0]
    h, h_o = act(rnd(M, W, seed=5), where)
    want = O.moe(h_o, cfg, sd, "")
    for fused in (True, False):
        x = torch.zeros((M, W), dtype=torch.float32, device=where[0])
        # the residual sum takes what the feed-forward returns
        ops.residual_norms(x, [torch.ones(W, device=where[0])], 1e-5, 1, dtype=where[1], **mod(h, fused))
        assert rel_err(x, want) < (where[2] if where[1] == torch.float32 else 4e-2), fused


@pytest.mark.parametrize("where", WHERE[:2])
def test_few_tokens_of_many_experts(where):
    """More pairs than experts, one expert that every token uses, experts nobody uses."""
    E, M, W, dt, dev = 8, 64, 64, torch.bfloat16 if where[0] == "cuda" else torch.float32, where[0]
    mod, cfg, sd = experts_module((dev, dt, 0), W, E, 3, 16, 1.0, 1.0, 1, 1, 8, 1.0)
    h, h_o = act(rnd(M, W, seed=5), (dev, dt))
    h_o[:, 0] = 4.0
    for e, v in enumerate((9.0, -9.0, 0.0, 0.0, -9.0, 0.5, 0.0, 1.0)):   # expert 0 always, 1 and 4 never
        sd["router"][e, 0] = v
    h = h_o.to(dt).to(dev)
    mod.router.weight.data[:E] = sd["router"].to(dt)
    x = torch.zeros((M, W), dtype=torch.float32, device=dev)
    ops.residual_norms(x, [torch.ones(W, device=dev)], 1e-5, 1, dtype=dt, **mod(h))
    assert rel_err(x, O.moe(h_o, cfg, sd, "")) < (2e-5 if dev == "cpu" else 4e-2)


# ------------------------------------------------------------------ generalised delta rule
def delta_case(where, B, T, H, D, rank, seed=0, strong=0.0):
    sz = ops.ChannelDeltaSizes(H, D, rank)
    n = (sz.columns + 15) // 16 * 16
    proj, proj_o = act(rnd(B, T, n, seed=seed), where)
    w2, w2_o = act(rnd(H * D, rank, seed=seed + 1) * 1.5 * rank ** -0.5, where)
    w0 = rnd(H * D, seed=seed + 2, mean=-2.0 + strong).float()
    ab = rnd(H * D, seed=seed + 3, std=0.5).float()
    norm = rnd(H * D, seed=seed + 4, std=0.2, mean=1.0).float()
    return sz, proj, proj_o, w2, w2_o, w0, ab, norm


def delta_oracle(case, b, T, eps, scale):
    """The first T tokens of sequence b -> [T, H D]."""
    sz, _, proj, _, w2, w0, ab, norm = case
    H, D, W = sz.heads, sz.dim, sz.width
    x = proj[b, :T]
    part = lambda i: x[:, i * W:(i + 1) * W].reshape(T, H, D)  # noqa: E731
    w = O.decay_of(x[:, 5 * W:5 * W + sz.rank], w2, w0.double()).view(T, H, D)
    a = torch.sigmoid(part(4) + ab.double().view(H, D))
    o, _ = O.delta_scan(part(0), part(1), part(2), w, a)
    return O.rms_normalise(o, eps).reshape(T, W) * norm.double() * torch.sigmoid(part(3).reshape(T, W)) * scale


def run_delta(where, case, cuts, lengths, slots, state, chunk_from, eps=1e-5, scale=0.7):
    sz, proj, _, w2, _, w0, ab, norm = case
    B, T, n = proj.shape
    d = where[0]
    outs, t0 = [], 0
    for c in cuts:
        left = (torch.tensor(lengths) - t0).clamp(0, c).to(torch.int32)
        full = bool((left == c).all())
        y = torch.full((B * c, sz.width + 8), 3.0, dtype=where[1], device=d)
        ops.channel_delta(proj[:, t0:t0 + c].reshape(B * c, n).contiguous(), B, c, sz, w2, w0.to(d), ab.to(d), norm.to(d), eps,
                          torch.full((B,), t0, dtype=torch.long, device=d), None if full else left.to(d), slots.to(d), state,
                          y[:, :sz.width], scale, chunk_from)
        assert bool((y[:, sz.width:] == 3.0).all())
        outs.append(y[:, :sz.width].reshape(B, c, -1))
        t0 += c
    return torch.cat(outs, 1)


def stale_state(where, slots, sz, value=5.0):
    state = torch.full((slots, sz.heads, sz.dim, sz.padded_dim), value, device=where[0])
    state[..., sz.dim:] = 0
    return state


SIZES = [(1, 8, 1), (3, 20, 7), (2, 33, 70), (2, 56, 12), (1, 64, 64), (2, 72, 130), (1, 128, 32), (1, 136, 9), (1, 250, 3)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,D,rank", SIZES)
def test_channel_delta(where, H, D, rank):
    """Two sequences of different lengths, whole (in chunks and token by token), in portions of several sizes
    and decoded one by one; slots that held something else before."""
    B, T, lens = 2, 75, [75, 41]
    case = delta_case(where, B, T, H, D, rank)
    sz = case[0]
    want = [delta_oracle(case, b, lens[b], 1e-5, 0.7) for b in range(B)]
    slots = torch.tensor([2, 0], dtype=torch.int32)
    plans = [([75], 16), ([75], 1000), ([2, 64, 1, 1, 7], 32), ([33, 2, 40], 2)]
    for cuts, chunk_from in plans[::3] if where[0] == "cpu" else plans:
        state = stale_state(where, 3, sz)
        got = run_delta(where, case, cuts, lens, slots, state, chunk_from)
        for b in range(B):
            assert rel_err(got[b, :lens[b]], want[b]) < where[2], (cuts, chunk_from, b)
            assert bool((got[b, lens[b]:] == 0).all())   # padding: a defined input of the projection
        assert bool((state[1, ..., :D] == 5.0).all())    # another's slot


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("strong", [-8.0, 8.0])
@pytest.mark.parametrize("D", [24, 80])
def test_channel_delta_weak_and_strong_decay(where, strong, D):
    """A state that hardly forgets (sums over hundreds of tokens), and one that forgets as fast as it can:
    every factor of a chunk is at its largest."""
    T = 330
    case = delta_case(where, 1, T, 2, D, 6, seed=9, strong=strong)
    want = delta_oracle(case, 0, T, 1e-5, 1.0)
    for cuts in ([T], [100, T - 100]):
        got = run_delta(where, case, cuts, [T], torch.zeros(1, dtype=torch.int32), stale_state(where, 1, case[0]), 16, scale=1.0)
        assert rel_err(got[0], want) < where[2] * 2


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("cuts", [[1] * 12, [5] + [1] * 7, [70] + [1] * 5])
def test_channel_delta_decode(where, cuts):
    """The first tokens one by one, and single tokens after a prompt; the slot's last owner leaves nothing."""
    T = sum(cuts)
    case = delta_case(where, 2, T, 4, 24, 9, seed=3)
    state = stale_state(where, 2, case[0], 2.0)
    for _ in range(2):
        got = run_delta(where, case, cuts, [T, T], torch.tensor([1, 0], dtype=torch.int32), state, 32)
        for b in range(2):
            assert rel_err(got[b], delta_oracle(case, b, T, 1e-5, 0.7)) < where[2]


def test_decay_is_bounded_and_both_terms_read_the_old_state():
    w = O.decay_of(rnd(50, 4, std=30.0), rnd(6, 4, seed=1, std=30.0), rnd(6, seed=2, std=9.0))
    assert float(w.min()) >= math.exp(-math.exp(-0.5)) - 1e-12 and float(w.max()) <= 1.0
    k, v, one = rnd(2, 1, 4), rnd(2, 1, 4, seed=1), torch.ones(2, 1, 4, dtype=torch.float64)
    k[1] = k[0]
    o, S = O.delta_scan(O.unit(k), k, v, one * 0.5, one, None)
    # second token: u^T S_1 removed from a state decayed by a half: - 1/2 k v_0 stays, k v_1 comes
    assert torch.allclose(S[0], torch.outer(k[0, 0], v[1, 0] - 0.5 * v[0, 0]), atol=1e-5)


# ------------------------------------------------------------------ attention: window and pooled blocks
class Attn:
    """One attention layer's inputs for B sequences of T tokens, and the oracle on them."""

    def __init__(self, where, B, T, H, G, D, window, pool, cap=None, scale=0.4, seed=0):
        self.where, self.B, self.T = where, B, T
        self.sz, self.rule = ops.PooledSizes(H, G, D), ops.PooledRule(scale, window, pool, 1e-5)
        self.n = (self.sz.columns + 15) // 16 * 16
        self.buf_o = rnd(B, T, self.n, seed=seed)
        self.qn, self.kn = rnd(H * D, seed=seed + 2, std=0.3, mean=1.2).float(), rnd(G * D, seed=seed + 3, std=0.3, mean=1.2).float()
        cap = min(cap or max(window, pool) + 15, T)
        z = lambda s, n: torch.full((s, G, n, D), 7.0, dtype=where[1], device=where[0])  # noqa: E731  (stale contents)
        self.cache = {"k": z(B + 1, cap), "v": z(B + 1, cap), "pk": z(B + 1, max(1, T // pool)), "pv": z(B + 1, max(1, T // pool)),
                      "tickets": torch.zeros((B + 1) * H, dtype=torch.int32, device=where[0])}
        self.slots = torch.arange(B, 0, -1, dtype=torch.int32, device=where[0])
        self.round()

    def round(self):   # after a change of the inputs
        self.buf, self.buf_o = act(self.buf_o, self.where)

    def step(self, t0, n, prompt, lengths=None, fused=True, decode=False, out_scale=0.6):
        d, B = self.where[0], self.B
        buf = self.buf[:, t0:t0 + n].reshape(B * n, self.n).clone()
        pos = torch.full((B, 1), t0, dtype=torch.long, device=d)
        lens = torch.tensor(lengths, dtype=torch.int32, device=d) if lengths is not None else None
        y = torch.full((B * n, self.sz.q_columns + 8), 3.0, dtype=self.where[1], device=d)
        out = y[:, :self.sz.q_columns]
        qn, kn = self.qn.to(d), self.kn.to(d)
        if decode:
            ops.pooled_decode(buf, self.sz, self.rule, qn, kn, pos, self.slots, self.cache, out, out_scale)
            assert int(self.cache["tickets"].abs().sum()) == 0
        else:
            keys = ops.pooled_prep_(buf, B, n, self.sz, self.rule, qn, kn, pos, lens, self.slots, self.cache, prompt)
            ops.pooled_attention(buf, keys, B, n, self.sz, self.rule, pos, lens, self.slots, self.cache, prompt, out, out_scale, fused)
        assert bool((y[:, self.sz.q_columns:] == 3.0).all())
        return out.reshape(B, n, -1)

    def oracle(self, b, T, window=None, pool=None, out_scale=0.6):
        sz, r = self.sz, self.rule
        H, G, D = sz.as_list()
        x = self.buf_o[b, :T, :sz.columns]
        v = x[:, H * D:].reshape(T, G, D)
        q = (O.rms_normalise(x[:, :H * D], r.eps) * self.qn.double()).view(T, H, D)
        k = (O.rms_normalise(x[:, H * D:], r.eps) * self.kn.double()).view(T, G, D)
        heads = [O.pooled_attention(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], r.scale, window or r.window, pool or r.pool)
                 for h in range(H)]
        return torch.cat(heads, -1) * out_scale

    def tol(self):
        return self.where[2] if self.where[1] != torch.bfloat16 else 4e-2   # bf16: q and k are rounded after their norms


ATTN = [  # H, G, D, window, pool
    (4, 2, 16, 37, 6), (2, 1, 40, 64, 16), (3, 3, 10, 1, 1), (2, 2, 72, 90, 90), (6, 1, 8, 3, 5), (2, 1, 128, 33, 64),
    (4, 4, 64, 128, 12), (1, 1, 136, 20, 7), (5, 1, 33, 200, 3), (8, 2, 24, 16, 130)]


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,window,pool", ATTN)
def test_pooled_attention(where, H, G, D, window, pool):
    """Prompts (matrix-core and row kernels) of unequal lengths, then portions, then decoding over a ring that
    wraps, against the oracle."""
    B, T = 2, 170
    a = Attn(where, B, T, H, G, D, window, pool)
    want, tol = [a.oracle(b, T) for b in range(B)], a.tol()
    for fused in (False, True) if where[0] == "cuda" else (True,):
        lens = [140, 97]
        got = a.step(0, 140, True, lens, fused=fused)
        for b in range(B):
            assert rel_err(got[b, :lens[b]], want[b][:lens[b]]) < tol, fused
            assert bool((got[b, lens[b]:] == 0).all())
        a.step(0, 140, True, None, fused=fused)
        t = 140
        for n in (2, 7, 14):
            got = a.step(t, n, False, None, fused=fused)
            for b in range(B):
                assert rel_err(got[b], want[b][t:t + n]) < tol, (fused, n)
            t += n
        for decode in (True, False, True, True, True):
            got = a.step(t, 1, False, None, fused=fused, decode=decode)
            for b in range(B):
                assert rel_err(got[b], want[b][t:t + 1]) < tol, (fused, "decode", decode)
            t += 1
        assert all(bool((a.cache[n][0] == 7.0).all()) for n in ("k", "v", "pk", "pv"))   # nobody's slot


def one_key_matches(a, at):
    """Only token `at`'s key has the component that all queries consist of: every other score is exactly zero,
    in 16 bits as well, whatever the values are."""
    H, G, D = a.sz.as_list()
    a.qn.fill_(1.0)
    a.kn.fill_(1.0)
    a.buf_o[0, :, :H * D] = 0
    a.buf_o[0, :, :H * D:D] = 1.0
    a.buf_o[0, :, H * D::D] = 0
    a.buf_o[0, at, H * D:(H + G) * D] = 0
    a.buf_o[0, at, H * D:(H + G) * D:D] = 3.0
    a.round()


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("window,pool", [(1, 2), (5, 5), (63, 8), (64, 7), (65, 1), (30, 50)])
def test_window_and_block_edges(where, window, pool):
    """One token's key outweighs all others for every query: seen alone while it is in the window, not at all
    until its block has left, then through the block's mean.  Prompts, portions and decoding; a window or a
    block one token off would change the output completely."""
    T, D, at = 190, 16, 41
    a = Attn(where, 1, T, 1, 1, D, window, pool, scale=0.75 * pool, seed=5)
    one_key_matches(a, at)
    want, tol = a.oracle(0, T), a.tol()
    edge = at + window                                           # the first query that has lost the token
    seen = (at // pool + 1) * pool - 1 + window                  # the first that sees its block
    assert blocks_seen(seen, a.rule) == at // pool + 1 and blocks_seen(seen - 1, a.rule) == at // pool
    assert rel_err(a.oracle(0, T, window + 1)[edge:edge + 1], want[edge:edge + 1]) > 0.2 or seen == edge
    if window > 1:
        assert rel_err(a.oracle(0, T, window - 1)[edge - 1:edge], want[edge - 1:edge]) > 0.2 or pool == 1
    if seen > edge:
        assert rel_err(a.oracle(0, T, window + 1)[seen:seen + 1], want[seen:seen + 1]) > 0.2
    assert rel_err(a.step(0, T, True)[0], want) < tol
    a.step(0, at - 2, True)
    for t in range(at - 2, min(T, seen + 3)):
        assert rel_err(a.step(t, 1, False, decode=t % 3 != 0)[0], want[t:t + 1]) < tol, t
    for cut in (2, 3, 11):
        a.step(0, 7, True)
        for t in range(7, T, cut):
            n = min(cut, T - t)
            assert rel_err(a.step(t, n, False)[0], want[t:t + n]) < tol, (cut, t)


@pytest.mark.parametrize("where", WHERE)
def test_first_tokens_see_only_what_is_there(where):
    """Sequences of one to seven tokens, prompt and decode, over a cache full of another sequence's keys and
    blocks."""
    a = Attn(where, 2, 8, 4, 2, 16, 3, 2, cap=52)
    want = [a.oracle(b, 8) for b in range(2)]
    for first in (1, 2, 5):
        got = a.step(0, first, True)
        for b in range(2):
            assert rel_err(got[b], want[b][:first]) < a.tol()
        for t in range(first, 8):
            got = a.step(t, 1, False, decode=True)
            for b in range(2):
                assert rel_err(got[b], want[b][t:t + 1]) < a.tol()


@pytest.mark.parametrize("where", WHERE)
def test_far_block_in_long_decoding(where):
    """The only matching key is hundreds of tokens back, in one of very many blocks."""
    T, D = 700, 24
    a = Attn(where, 1, T, 2, 1, D, 10, 4, scale=2.5, seed=7)
    one_key_matches(a, 13)
    want = a.oracle(0, T)
    away = a.buf_o.clone()
    a.buf_o[0, 13] *= -1
    assert rel_err(a.oracle(0, T)[-3:], want[-3:]) > 0.2   # the far key is what decides
    a.buf_o = away
    a.step(0, T - 4, True)
    for t in range(T - 4, T):
        assert rel_err(a.step(t, 1, False, decode=True)[0], want[t:t + 1]) < a.tol()


@pytest.mark.gpu
@pytest.mark.parametrize("window,pool,T", [(63, 2, 300), (64, 1, 400), (255, 3, 700), (1200, 16, 2600)])
@pytest.mark.parametrize("heads,dim", [(2, 12), (4, 24)])   # any-size kernel; four heads a workgroup
def test_split_decode(window, pool, T, heads, dim):
    """Decoding over many visible keys (several workgroups per head and a merge), repeated."""
    where = ("cuda", torch.float32, 5e-5)
    a = Attn(where, 1, T, heads, 1, dim, window, pool, scale=1.0, seed=8)
    want = a.oracle(0, T)
    a.step(0, T - 5, True)
    for t in range(T - 5, T):
        assert rel_err(a.step(t, 1, False, decode=True)[0], want[t:t + 1]) < where[2]


@pytest.mark.gpu
@pytest.mark.parametrize("B,H,G", [(16, 8, 2), (40, 8, 2), (48, 6, 3)])
def test_decode_shares_keys_between_heads(B, H, G):
    """Enough sequences that several query heads of a key / value head share a workgroup, against the
    one-wave-a-query kernel on the same cache; some sequences are much shorter than the window."""
    where = ("cuda", torch.float32, 5e-5)
    a = Attn(where, B, 150, H, G, 24, 60, 7, cap=150, seed=12)
    a.step(0, 149, True)
    pos = torch.randint(0, 150, (B, 1), generator=torch.Generator().manual_seed(3)).cuda()
    buf = a.buf[:, 149].contiguous()
    other = {n: t.clone() for n, t in a.cache.items()}
    got, want = (torch.empty(B, H * 24, device="cuda") for _ in range(2))
    ops.pooled_decode(buf, a.sz, a.rule, a.qn.cuda(), a.kn.cuda(), pos, a.slots, other, got)
    row = buf.clone()
    kn = ops.pooled_prep_(row, B, 1, a.sz, a.rule, a.qn.cuda(), a.kn.cuda(), pos, None, a.slots, a.cache, False)
    ops.pooled_attention(row, kn, B, 1, a.sz, a.rule, pos, None, a.slots, a.cache, False, want, fused=False)
    assert rel_err(got, want.cpu()) < 5e-5
    for n in ("k", "v", "pk", "pv"):
        assert rel_err(other[n].flatten(0, 2), a.cache[n].flatten(0, 2).cpu()) < 1e-5
    assert int(other["tickets"].abs().sum()) == 0


@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 5, 8, 16])
@pytest.mark.parametrize("N,K", [(48, 72), (33, 8), (200, 2048), (1000, 1000), (16, 4096)])
def test_products_of_some_rows(M, N, K):
    w, x = (rnd(N, K) * K ** -0.5).bfloat16(), rnd(M, K, seed=1).bfloat16()
    assert rel_err(ops.linear_few(x.cuda(), w.cuda()), x.double() @ w.double().T) < 8e-3


@pytest.mark.gpu
@pytest.mark.parametrize("M", [1, 3, 4])
def test_scaled_logits_of_a_few_rows(M):
    w, x = (rnd(77, 48) * 48 ** -0.5).bfloat16(), rnd(M, 48, seed=1).bfloat16()
    y = ops.decode_linear(w.cuda(), x.cuda(), epilogue="f32", alpha=0.3)
    assert rel_err(y, x.double() @ w.double().T * 0.3) < 1e-4


# ------------------------------------------------------------------ both side by side
@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("H,G,D,R,E,rank", [(3, 1, 10, 2, 9, 5), (4, 2, 16, 2, 32, 8)])
def test_parallel_mixer(where, H, G, D, R, E, rank):
    W, T, eps, dev, dt = 40, 50, 1e-5, where[0], where[1]
    mix = ParallelMixer(W, PooledAttention(H, G, D, 0.4, 11, 4, eps, dev), ChannelDelta(R, E, rank, eps, dt, dev), 0.5, 1.5, dt, dev)
    n = R * E
    sd = {"left.q": (H * D, W), "left.k": (G * D, W), "left.o": (W, H * D), "right.w1": (rank, W), "right.w2": (n, rank), "right.o": (W, n)}
    sd.update({f"right.{x}": (n, W) for x in "rkvga"})
    sd = {k: (rnd(*s, seed=i) * s[1] ** -0.5).to(dt).double() for i, (k, s) in enumerate(sd.items())}
    for i, (k, c) in enumerate((("left.q.norm", H * D), ("left.k.norm", G * D), ("right.w0", n), ("right.a.b", n), ("right.norm", n))):
        sd[k] = rnd(c, seed=40 + i, std=0.3, mean=1.0).float().double()
    ip, op = mix.in_proj.weight.data.zero_(), mix.o_proj.weight.data.zero_()
    left, right = torch.cat([sd["left.q"], sd["left.k"]]), torch.cat([sd[f"right.{x}"] for x in ("r", "k", "v", "g", "a", "w1")])
    ip[:left.shape[0]] = left.to(dt)
    ip[mix.in_split:mix.in_split + right.shape[0]] = right.to(dt)
    op[:, :H * D] = sd["left.o"].to(dt)
    op[:, mix.out_split:mix.out_split + n] = sd["right.o"].to(dt)
    for t, k in ((mix.left.q_norm, "left.q.norm"), (mix.left.k_norm, "left.k.norm"), (mix.right.w2, "right.w2"),
                 (mix.right.w0, "right.w0"), (mix.right.a_bias, "right.a.b"), (mix.right.out_norm, "right.norm")):
        t.data.copy_(sd[k])
    for p in mix.parameters():
        p.requires_grad_(False)
    h, h_o = act(rnd(T, W, seed=60), where)
    m = {"left": {"heads": H, "kv_heads": G, "dim": D, "scale": 0.4, "mask": {"size": 11, "pool": 4}}, "left_scale": 0.5,
         "right": {"heads": R, "dim": E}, "right_scale": 1.5}
    want = O.parallel_mixer(h_o, m, sd, "", eps)
    cache = mix.cache_tensors(2, 64, dt, dev)
    slots = torch.tensor([1], dtype=torch.int32, device=dev)
    got = []
    for t0, t1 in ((0, 30), (30, 32), (32, 45)) + tuple((t, t + 1) for t in range(45, T)):
        pos = torch.arange(t0, t1, device=dev)[None]
        got.append(mix(h[t0:t1], cache, StepContext(1, t1 - t0, pos, None, slots, t0 == 0, dev == "cuda")))
    assert rel_err(torch.cat(got), want) < (where[2] if dt == torch.float32 else 5e-2)
