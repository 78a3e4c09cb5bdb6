"""The Bezurax model through the framework's own loader, registry, cache, batch sessions and generate(),
against the plain implementation in bezurax_oracle.py (CPU: the package's reference operations; GPU: the
HIP kernels in fp32 and bf16)."""

import io
import json
import os
import subprocess
import sys

import pytest
import torch

import bezurax_oracle as O
from bezurax_cases import CONFIGS, RANKS, config, layer, mixer, moe
from bezurax_cases import weights as random_weights
from golitar_cases import doubles, rel_err, row_errs, tokens, write_model
from neuronx_distributed_llama3_2_amd.inference import (BatchSession, BezuraxForCausalLMInference, BezuraxRunner,
                                                        InferenceConfig, app_class, runner_class)
from neuronx_distributed_llama3_2_amd.inference.registry import family_name
from neuronx_distributed_llama3_2_amd.inference.trace_replay import replay
from neuronx_distributed_llama3_2_amd.models.bezurax import BezuraxConfig

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.mark.gpu
# (device, dtype); the CPU variants stay on the CPU also where a GPU is visible
WHERE = [pytest.param((torch.device("cpu"), torch.float32), id="cpu"),
         pytest.param((torch.device("cuda", 0), torch.float32), id="gpu-fp32", marks=GPU),
         pytest.param((torch.device("cuda", 0), torch.bfloat16), id="gpu-bf16", marks=GPU)]


def weights(name, seed=0):
    return random_weights(CONFIGS[name], seed, RANKS[name])


def logits_agree(got, want, dtype):
    """fp32: every row within 3e-4.  bf16: a close call between two experts goes either way within rounding and
    moves the rows it happens in, so the average and nearly all rows are what is held small."""
    e = row_errs(got, want)
    if dtype == torch.float32:
        return float(e.max()) < 3e-4
    return float(e.mean()) < 5e-2 and float((e > 0.25).double().mean()) < 0.1


_ORACLE = {}


def oracle_logits(name, toks, seed=0):
    key = (name, tuple(toks), seed)
    if key not in _ORACLE:
        _ORACLE[key] = O.forward(CONFIGS[name], doubles(weights(name, seed)), toks)
    return _ORACLE[key]


def make_app(path, device, dtype, max_len=256, batch=4, **kw):
    kw.setdefault("enable_bucketing", True)
    cfg = InferenceConfig(batch_size=batch, seq_len=max_len, **kw)
    mc = BezuraxConfig.from_pretrained(path)
    app = BezuraxForCausalLMInference(mc, cfg, dtype, device=device, init_weights=False)
    from neuronx_distributed_llama3_2_amd.inference.generation import load_hf_state_dict

    app._load_full(app._hf_to_nxd(load_hf_state_dict(path), mc))
    return app


@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    out = {}
    for name, cfg in CONFIGS.items():
        out[name] = write_model(tmp_path_factory.mktemp(name), cfg, weights(name))
    return out


NAMES = sorted(CONFIGS)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_portions_and_decoding(where, name, model_dirs):
    """One sequence: the whole prompt in one step; the prompt cut at several places (down to two tokens);
    most of it decoded token by token."""
    device, dtype = where
    T = 120
    toks = tokens(T, CONFIGS[name]["vocab"])
    want = oracle_logits(name, toks)
    app = make_app(model_dirs[name], device, dtype)
    s = BatchSession(app)
    assert logits_agree(s.step([("a", toks, range(T))]), want, dtype)
    s.end(["a"])
    got = [s.step([("a", toks[:40], range(40))])]
    for t in range(40, T):
        got.append(s.step([("a", [toks[t]], [0])]))
    assert logits_agree(torch.cat(got), want, dtype)
    s.end(["a"])
    # several new tokens at a time over the cache (the step function's general form)
    for first, cut in ((1, 2), (30, 16), (50, 70)):
        ids = torch.tensor([toks], device=device)
        pos = torch.arange(T, device=device).unsqueeze(0)
        slot = torch.tensor([2], device=device)
        fwd = app.model.forward_tokens
        got = [fwd(ids[:, :first], pos[:, :first], slot, prefill=True)[0]]
        for t in range(first, T, cut):
            got.append(fwd(ids[:, t:t + cut], pos[:, t:t + cut], slot)[0])
        assert logits_agree(torch.cat(got), want, dtype), (first, cut)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["mixed", "plain"])
def test_batches_of_unequal_requests(where, name, model_dirs):
    """Requests of different lengths together, each leaving as it ends, against each alone; then another
    batch in the slots they have left."""
    device, dtype = where
    app = make_app(model_dirs[name], device, dtype)
    s = BatchSession(app)
    V = CONFIGS[name]["vocab"]
    for rnd, plan in enumerate(({"a": (1, 4), "b": (33, 12), "c": (90, 8), "d": (7, 15)}, {"e": (64, 9), "f": (2, 5)})):
        seqs = {r: tokens(p + d, V, seed=10 * rnd + i) for i, (r, (p, d)) in enumerate(plan.items())}
        want = {r: oracle_logits(name, t) for r, t in seqs.items()}
        out = s.step([(r, seqs[r][:p], range(p)) for r, (p, _) in plan.items()])
        got = dict(zip(plan, torch.split(out, [p for p, _ in plan.values()])))
        done = 0
        live = list(plan)
        while live:
            out = s.step([(r, [seqs[r][plan[r][0] + done]], [0]) for r in live])
            for r, row in zip(live, out):
                got[r] = torch.cat([got[r], row[None]])
            done += 1
            gone = [r for r in live if plan[r][1] == done]
            s.end(gone)
            live = [r for r in live if r not in gone]
        for r in plan:
            assert logits_agree(got[r], want[r], dtype), r
    assert s._free == list(range(app.max_batch))


@pytest.mark.parametrize("where", WHERE)
def test_long_decoding(where, tmp_path):
    """Decoding far past every window, so that the key rings wrap several times and most of what is seen are
    blocks; two layers share their weights and nothing else."""
    device, dtype = where
    name = "long"
    first = layer(mixer(window=17, pool=4, rheads=2, rdim=12), None)
    CONFIGS[name] = config([first, layer(mixer(window=66, pool=30), moe(experts=4, groups=(2, 1), ff=16)), dict(first, weights_of=0)],
                           width=48, vocab=71)
    toks = tokens(300 if device.type == "cuda" else 200, 71)
    want = oracle_logits(name, toks)
    app = make_app(write_model(tmp_path / "m", CONFIGS[name], weights(name)), device, dtype, max_len=len(toks), batch=1)
    caches = [app.model.kv_cache[i] for i in range(3)]
    assert caches[0]["k"].shape[2] == 64   # one window and some, not the whole sequence
    assert caches[0]["state"].data_ptr() != caches[2]["state"].data_ptr() and caches[0]["k"].data_ptr() != caches[2]["k"].data_ptr()
    assert len(app.model.model.layers) == 2
    s = BatchSession(app)
    got = [s.step([("a", toks[:3], range(3))])]
    for t in range(3, len(toks)):
        got.append(s.step([("a", [toks[t]], [0])]))
    assert logits_agree(torch.cat(got), want, dtype)


def greedy(name, prompt, n, seed=0):
    W, cfg, toks = doubles(weights(name, seed)), CONFIGS[name], list(prompt)
    for _ in range(n):
        toks.append(int(O.forward(cfg, W, toks)[-1].argmax()))
    return toks


@pytest.mark.parametrize("where", WHERE[:2])
def test_greedy_generation(where, model_dirs):
    """generate(): right-padded prompts of different lengths, greedy, decode graphs on the GPU.  Twice with
    the same application: the second call finds captured graphs and used slots."""
    name = "mixed"
    app = make_app(model_dirs[name], where[0], where[1], max_len=64, decode_graph_steps=4)
    V = CONFIGS[name]["vocab"]
    prompts = [tokens(9, V, seed=21), tokens(17, V, seed=22)]
    ids = torch.zeros((2, 17), dtype=torch.long)
    mask = torch.zeros((2, 17), dtype=torch.long)
    for i, p in enumerate(prompts):
        ids[i, :len(p)] = torch.tensor(p)
        mask[i, :len(p)] = 1
    want = [greedy(name, p, 10)[len(p):] for p in prompts]
    for _ in range(2):
        out = app.generate(ids, mask, max_new_tokens=10).cpu()
        assert [out[i, 17:].tolist() for i in range(2)] == want


@pytest.mark.gpu
@pytest.mark.parametrize("graphs", [True, False])
def test_generation_bf16(graphs, model_dirs):
    """bf16: every generated token has the largest logit, or one within rounding of it, when the same
    tokens are fed step by step; captured graphs and eager steps, replays after the first."""
    device = torch.device("cuda", 0)
    app = make_app(model_dirs["wide_heads"], device, torch.bfloat16, max_len=200, decode_graph_steps=8, use_hip_graphs=graphs)
    V = CONFIGS["wide_heads"]["vocab"]
    prompts = torch.tensor([tokens(40, V, seed=31), tokens(40, V, seed=32)])
    out = app.generate(prompts, max_new_tokens=100, eos_token_id=-1).cpu()
    s = BatchSession(app)
    logits = [s.step([("a", out[0, :40].tolist(), [39]), ("b", out[1, :40].tolist(), [39])])]
    for t in range(40, 139):
        logits.append(s.step([("a", [int(out[0, t])], [0]), ("b", [int(out[1, t])], [0])]))
    logits = torch.stack(logits, 1).float().cpu()   # [2, 100, V]
    chosen = logits.gather(2, out[:, 40:].unsqueeze(-1)).squeeze(-1)
    assert float((logits.max(-1).values - chosen).max()) < 0.1


@pytest.mark.gpu
def test_sampling(model_dirs):
    app = make_app(model_dirs["mixed"], torch.device("cuda", 0), torch.bfloat16, max_len=96)
    ids = torch.tensor([tokens(20, CONFIGS["mixed"]["vocab"])])
    a = app.generate(ids, max_new_tokens=30, do_sample=True, top_k=8, temperature=1.2, seed=5)
    b = app.generate(ids, max_new_tokens=30, do_sample=True, top_k=8, temperature=1.2, seed=5)
    c = app.generate(ids, max_new_tokens=30, do_sample=True, top_k=8, temperature=1.2, seed=6)
    assert torch.equal(a, b) and not torch.equal(a, c)


@pytest.mark.gpu
def test_fused_decode_switch(model_dirs):
    """set_fused_decode(False) takes the unfused operations: the same logits up to rounding."""
    app = make_app(model_dirs["wide_heads"], torch.device("cuda", 0), torch.bfloat16)
    toks = tokens(60, CONFIGS["wide_heads"]["vocab"])
    outs = []
    for on in (True, False):
        app.set_fused_decode(on)
        s = BatchSession(app)
        o = [s.step([("a", toks[:30], range(30))])]
        o += [s.step([("a", [t], [0])]) for t in toks[30:]]
        outs.append(torch.cat(o))
        s.end(["a"])
    assert logits_agree(outs[0], outs[1].cpu(), torch.bfloat16)


def test_registry_and_runner(model_dirs, tmp_path):
    path = model_dirs["mixed"]
    assert app_class(path) is BezuraxForCausalLMInference and runner_class(path) is BezuraxRunner
    assert family_name({"architectures": ["LlamaForCausalLM"], "model_type": "llama"}) == "llama"
    assert family_name({"architectures": ["MixtralForCausalLM"]}) == "mixtral"
    with pytest.raises(ValueError):
        family_name({"architecture": "SomethingElse"})
    r = BezuraxRunner(path)
    m = r.load_neuron_model_on_cpu(16, 32, 1)
    if m.device.type == "cpu":
        out = r.generate_on_neuron([tokens(8, 211)], m, max_length=14)
        assert out[0].tolist() == greedy("mixed", tokens(8, 211), 6)


def test_compile_and_load(model_dirs, tmp_path):
    """The compiled form (framework names, per-rank file) serves the same logits."""
    device = torch.device("cpu")
    app = make_app(model_dirs["mixed"], device, torch.float32, batch=1)
    app.compile(str(tmp_path / "c"))
    toks = tokens(25, 211)
    a = BatchSession(app).step([("x", toks, range(25))])
    assert app_class(str(tmp_path / "c")) is BezuraxForCausalLMInference
    if torch.cuda.is_available():
        return   # load() picks the GPU there; covered by the bf16 test below
    again = BezuraxForCausalLMInference.load(str(tmp_path / "c"), dtype=torch.float32)
    assert torch.equal(a, BatchSession(again).step([("x", toks, range(25))]))


@pytest.mark.gpu
def test_runner_on_gpu(model_dirs, tmp_path):
    r = BezuraxRunner(model_dirs["wide_heads"])
    r.trace(str(tmp_path / "t"), batch_size=1, max_prompt_length=32, sequence_length=64)
    m = r.load_neuron_model(str(tmp_path / "t"))
    out = r.generate_on_neuron([tokens(20, 130)], m, max_length=40)
    assert out.shape == (1, 40)
    rep = r.benchmark_sampling(m, num_runs=2, report_path=str(tmp_path / "r.json"))
    assert rep["e2e_model"]["throughput"] > 0


def test_config_is_checked():
    base = CONFIGS["mixed"]

    def parse(change, rank=7):
        c = json.loads(json.dumps(base))
        for l in c["layers"]:
            l["mixer"]["right"]["rank"] = rank
        change(c)
        return BezuraxConfig(c)

    for change in (lambda c: c["layers"][0].__setitem__("type", "other"),
                   lambda c: c["layers"][3]["mlp"].__setitem__("kind", "dense"),
                   lambda c: c["layers"][3]["mixer"]["left"].__setitem__("kv_heads", 4),
                   lambda c: c["layers"][3]["mixer"]["left"].__setitem__("vdim", 12),
                   lambda c: c["layers"][3]["mlp"]["router"].__setitem__("top", 6),
                   lambda c: c["layers"][3]["mlp"]["router"].__setitem__("groups", {"count": 2, "keep": 1}),
                   lambda c: c["layers"][2].__setitem__("weights_of", 1),    # another layer's sizes
                   lambda c: c["layers"][2].__setitem__("weights_of", 2),
                   lambda c: c["norm"].__setitem__("groups", 7),
                   lambda c: c["layers"][3]["mixer"]["right"].pop("rank")):
        with pytest.raises(ValueError):
            parse(change)
    cfg = parse(lambda c: None)
    assert cfg.unique == [0, 1, 3] and cfg.use == [0, 1, 0, 2, 1] and cfg.layers[1].mlp is None
    assert cfg.layers[3].mlp.shared_ff == 0


def test_a_layer_may_use_a_later_ones_weights(tmp_path):
    """The tensors stand under the number of the layer that has them, wherever it is."""
    own = layer(mixer(heads=2, kv_heads=1, window=9, pool=2), moe())
    CONFIGS["later"], RANKS["later"] = config([dict(own, weights_of=2), layer(mixer(), None), own, dict(own, weights_of=2)], vocab=41), 3
    toks = tokens(60, 41)
    app = make_app(write_model(tmp_path, CONFIGS["later"], weights("later")), torch.device("cpu"), torch.float32, batch=1)
    got = BatchSession(app).step([("a", toks, range(60))])
    assert logits_agree(got, oracle_logits("later", toks), torch.float32)


def test_missing_weights_are_reported(tmp_path):
    sd = weights("mixed")
    del sd["l3.mlp.e2.up"]
    with pytest.raises(KeyError):
        make_app(write_model(tmp_path, CONFIGS["mixed"], sd), torch.device("cpu"), torch.float32)


def test_session_and_replay_errors(model_dirs):
    app = make_app(model_dirs["plain"], torch.device("cpu"), torch.float32, max_len=32, batch=1)
    s = BatchSession(app)
    toks = tokens(12, 53)
    with pytest.raises(ValueError):
        s.step([("a", toks, [12])])
    s.step([("a", toks[:5], []), ("b", toks[:3], [])])   # more requests than slots: the cache grows
    assert app.max_batch == 2
    for bad in ([("c", toks[:2], [])], [("a", toks[:2], [])], [("a", [1], []), ("a", [1], [])], [("a", [], [])]):
        with pytest.raises(ValueError):
            s.step(bad)
    s.end(["a", "b"])
    with pytest.raises(ValueError):
        s.step([("a", tokens(40, 53), [])])


def test_replay_writes_the_wanted_logits(model_dirs, tmp_path):
    name = "plain"
    app = make_app(model_dirs[name], torch.device("cpu"), torch.float32, max_len=64, batch=1)
    a, b = tokens(11, 53, seed=1), tokens(6, 53, seed=2)
    lines = [json.dumps({"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [8, 2]}, {"id": "b", "tokens": b[:5], "want": []}],
                         "end": []}),
             json.dumps({"step": 1, "entries": [{"id": "b", "tokens": b[5:], "want": [0]}, {"id": "a", "tokens": a[9:10], "want": []}],
                         "end": ["b"]}),
             json.dumps({"step": 2, "entries": [{"id": "a", "tokens": a[10:], "want": []}], "end": ["a"]})]
    out = io.StringIO()
    replay(BatchSession(app), lines, str(tmp_path), out)
    assert out.getvalue().split("\n")[:3] == ["done 0", "done 1", "done 2"]
    load = lambda n: torch.frombuffer(bytearray((tmp_path / n).read_bytes()), dtype=torch.float32).view(-1, 53)  # noqa: E731
    wa, wb = oracle_logits(name, a), oracle_logits(name, b)
    assert rel_err(load("0.f32"), wa[[8, 2]]) < 3e-4 and rel_err(load("1.f32"), wb[[5]]) < 3e-4
    assert not (tmp_path / "2.f32").exists()


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(dtype, model_dirs, tmp_path):
    name = "mixed"
    toks = tokens(30, 211, seed=4)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:28], "want": list(range(28))}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[28:29], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "q", "tokens": toks[29:], "want": [0]}], "end": ["q"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", model_dirs[name], "--dtype", dtype, "--out",
                        str(tmp_path), "--max-tokens", "30"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=110, env=dict(os.environ, HOME=str(tmp_path)))
    assert r.returncode == 0, r.stderr[-2000:]
    got = torch.cat([torch.frombuffer(bytearray((tmp_path / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, 211)
                     for i in range(3)])
    assert logits_agree(got, oracle_logits(name, toks), getattr(torch, dtype))


def test_trace_run_needs_a_gpu(model_dirs, tmp_path):
    """No CPU path behind the program."""
    env = dict(os.environ, HIP_VISIBLE_DEVICES="", CUDA_VISIBLE_DEVICES="")
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", model_dirs["mixed"], "--out", str(tmp_path),
                        "--max-tokens", "8"], input="", capture_output=True, text=True, timeout=600, env=env)
    assert r.returncode != 0 and "GPU" in r.stderr


def test_command_line(model_dirs, tmp_path, capsys):
    sys.path.insert(0, os.path.join(ROOT, "examples", "inference"))
    from llama3_2_runner import main

    out = str(tmp_path / "traced")
    main(["trace", "--model_path", model_dirs["mixed"], "--traced_path", out, "--max_prompt_length", "8", "--sequence_length", "14"],
         runner_cls=BezuraxRunner)
    rows = main(["generate", "--traced_path", out, "--prompt_ids", ",".join(map(str, tokens(8, 211)))], runner_cls=BezuraxRunner)
    assert rows.shape == (1, 14) and rows[0, :8].tolist() == tokens(8, 211)


def test_benchmark_configurations():
    """bench.py --serve: a token uses as many feed-forward parameters as in the Llama models beside it."""
    from neuronx_distributed_llama3_2_amd.inference.serve_bench import SIZES, bezurax_config

    for size, ff, layers in zip(SIZES, (8192, 14336), (16, 8)):
        cfg = BezuraxConfig(bezurax_config(size))
        m = cfg.layers[0].mlp
        assert m.top * m.ff + m.shared_ff == ff and cfg.num_hidden_layers == layers
