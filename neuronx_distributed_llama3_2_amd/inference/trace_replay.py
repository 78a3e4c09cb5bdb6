"""Replay of a token trace: JSON steps on standard input, logits as raw fp32 files (bin/trace_run).

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [0, 1]}], "end": []}

A step is one batch: whole prompts of new requests, or one token more for each of some running ones.
The logits at the wanted places go to <out>/<step>.f32 ([wanted, vocab], little-endian), then
"done <step>" is printed; requests in "end" give their cache slots back."""

from __future__ import annotations

import argparse
import json
import os
import sys

import torch

from .config import InferenceConfig
from .registry import app_class
from .session import BatchSession

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def build_session(model_dir: str, dtype: torch.dtype, max_tokens: int) -> BatchSession:
    if not torch.cuda.is_available():
        raise RuntimeError("trace replay runs on the GPU and none is visible")
    if dtype == torch.float32:
        torch.backends.cuda.matmul.allow_tf32 = False
        torch.set_float32_matmul_precision("highest")
    config = InferenceConfig(batch_size=1, seq_len=max(int(max_tokens), 1), enable_bucketing=True,
                             decode_graph_steps=1)
    return BatchSession(app_class(model_dir).from_pretrained(model_dir, config, dtype=dtype))


def replay(session: BatchSession, lines, out_dir: str, stdout) -> None:
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = session.step([(e["id"], e["tokens"], e["want"]) for e in step["entries"]])
        if logits is not None:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            logits.float().cpu().numpy().astype("<f4").tofile(path)
        session.end(step["end"])
        print(f"done {step['step']}", file=stdout, flush=True)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    a = ap.parse_args(argv)
    os.makedirs(a.out, exist_ok=True)
    session = build_session(a.model, DTYPES[a.dtype], a.max_tokens)
    replay(session, sys.stdin, a.out, sys.stdout)
    return 0
