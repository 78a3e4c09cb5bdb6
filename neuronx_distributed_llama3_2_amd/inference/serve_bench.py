"""Serving throughput of a model family at layer sizes of a real model (random weights, one GPU):
context encoding and token generation through the application's own captured graphs
(bench.py --serve FAMILY).

The Golitar sizes are built to equal the Llama ones: the same width, depth and vocabulary, the same
parameters in the feed-forward (two matrices instead of three), three gated-delta layers to one
differential-attention layer.  The Bezurax sizes have the same width, depth and vocabulary, heads as
Golitar's in both mixers of every layer, and the feed-forward parameters that a token uses equal to
Llama's (half of them in the shared expert, half in 4 of 32 routed ones)."""

from __future__ import annotations

import json
from typing import Dict, List, Optional

import torch

from .config import InferenceConfig

FAMILIES = ("bezurax", "golitar", "llama")
SIZES = ("2k", "4k")
# (sequences, tokens) of a prompt batch; sequences of a decode batch
PREFILL = [(1, 8192), (4, 2048), (1, 2048)]
DECODE = [1, 2, 8, 16, 32]
DECODE_CONTEXT = 2048


def golitar_config(size: str) -> dict:
    """config.json of the benchmark model of this size."""
    width, layers, ff, heads, kv = {"2k": (2048, 16, 12288, 16, 4), "4k": (4096, 8, 21504, 32, 8)}[size]
    mlp = {"kind": "dense", "ff": ff}
    delta = {"type": "delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4}}
    attn = {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": 64, "vdim": 128, "diff": 0.5, "scale": 0.125,
                      "softcap": 30.0, "mask": {"size": 1024},
                      "rot": {"dims": 32, "base": 500000.0,
                              "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}}
    return {"architecture": "Golitar", "layers": [attn if i % 4 == 3 else delta for i in range(layers)],
            "width": width, "vocab": 128256, "streams": 4, "norm": {"eps": 1e-5}, "logit_softcap": 30.0}


def bezurax_config(size: str) -> dict:
    """config.json of the benchmark model of this size."""
    width, layers, ff, heads, kv, rank = {"2k": (2048, 16, 1024, 16, 4, 64), "4k": (4096, 8, 1792, 32, 8, 96)}[size]
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": 4 * ff, "limit": 7.0},
           "router": {"experts": 32, "top": 4, "groups": {"count": 4, "keep": 2}, "scale": 2.5}}
    mixer = {"left": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                      "mask": {"size": 1024, "pool": 16}},
             "left_scale": 0.7, "right": {"heads": heads, "dim": 128, "rank": rank}, "right_scale": 0.7}
    return {"architecture": "Bezurax", "layers": [{"type": "parallel", "mixer": mixer, "mlp": mlp}] * layers,
            "width": width, "vocab": 128256, "norm": {"eps": 1e-5, "groups": 8}, "logit_scale": 1.0}


def build(family: str, size: str, batch: int, max_len: int, context: int):
    icfg = InferenceConfig(batch_size=batch, seq_len=max_len, max_context_length=context, decode_graph_steps=8)
    torch.manual_seed(0)
    if family == "golitar":
        from ..models.golitar import GolitarConfig
        from .golitar import GolitarForCausalLMInference

        return GolitarForCausalLMInference(GolitarConfig(golitar_config(size)), icfg)
    if family == "bezurax":
        from ..models.bezurax import BezuraxConfig
        from .bezurax import BezuraxForCausalLMInference

        return BezuraxForCausalLMInference(BezuraxConfig(bezurax_config(size)), icfg)
    from ..models.llama.modeling_llama import llama_config
    from .generation import LlamaForCausalLMInference

    cfg = llama_config("llama3.2-1b") if size == "2k" else llama_config("llama3-8b", num_hidden_layers=8)
    return LlamaForCausalLMInference(cfg, icfg)


def _time(fn, reps: int) -> float:
    """Milliseconds a call, between events on the device."""
    for _ in range(2):
        fn()
    start, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    torch.cuda.synchronize()
    start.record()
    for _ in range(reps):
        fn()
    end.record()
    torch.cuda.synchronize()
    return start.elapsed_time(end) / reps


def measure(family: str, size: str, steps: int, prefill=None, decode=None) -> Dict[str, list]:
    from ..utils.sampling import Sampler

    out: Dict[str, list] = {"prefill": [], "decode": []}
    for B, T in PREFILL if prefill is None else prefill:
        app = build(family, size, B, T, T)
        ids = torch.randint(10, app.model_config.vocab_size, (B, T))
        ms = _time(lambda: app._context_encode(ids), steps)
        out["prefill"].append({"batch": B, "tokens": T, "ms": round(ms, 3), "tokens_per_s": round(1000 * B * T / ms)})
        del app
        torch.cuda.empty_cache()
    for B in DECODE if decode is None else decode:
        app = build(family, size, B, DECODE_CONTEXT + 512, DECODE_CONTEXT)
        app.config.prefill_graphs = False
        ids = torch.randint(10, app.model_config.vocab_size, (B, DECODE_CONTEXT))
        first = app._context_encode(ids).argmax(-1)
        st = app._decode_state(B)
        st.load(first, torch.full((B,), DECODE_CONTEXT), torch.arange(B))
        g = app._graph(B, Sampler(None, top_k=1))
        ms = _time(g.replay, steps) / g.steps
        out["decode"].append({"batch": B, "context": DECODE_CONTEXT, "ms_per_step": round(ms, 4),
                              "tokens_per_s": round(1000 * B / ms)})
        del app, g, st
        torch.cuda.empty_cache()
    return out


def run(family: str, sizes: Optional[List[str]], steps: int, phase: str = "both") -> None:
    """One JSON line."""
    if not torch.cuda.is_available():
        raise SystemExit("bench --serve needs a GPU")
    torch.cuda.set_device(0)
    torch.set_grad_enabled(False)
    res = {}
    for size in sizes or SIZES:
        res[size] = measure(family, size, steps, [] if phase == "decode" else None, [] if phase == "prefill" else None)
    print(json.dumps({"metric": f"serving throughput, {family}", "unit": "tokens/s", "n_gpus": 1, "steps": steps,
                      "dtype": "bf16", "data": "synthetic (random token ids, random-init weights)", "sizes": res}),
          flush=True)
