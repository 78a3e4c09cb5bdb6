"""Golitar model configuration: the reader of its config.json.

A Golitar decoder is a list of layers; each names its mixer ("delta": gated delta rule, "attention":
differential attention with a sliding window), the mixer's sizes, and its feed-forward (dense, squared
ReLU) or none.  Several residual streams are mixed around every sublayer."""

from __future__ import annotations

import copy
import json
import os
from dataclasses import dataclass
from typing import Any, Dict, List, Optional

ARCHITECTURE = "Golitar"


@dataclass(frozen=True)
class DeltaMixerConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class RotaryConfig:
    dims: int
    base: float
    factor: Optional[float] = None     # None: no frequency scaling
    low: float = 1.0
    high: float = 4.0
    original: float = 8192.0


@dataclass(frozen=True)
class AttentionMixerConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    diff: float
    scale: float
    rot: RotaryConfig
    softcap: float = 0.0               # 0: none
    window: int = 0                    # 0: every earlier token


@dataclass(frozen=True)
class LayerConfig:
    type: str                          # "delta" | "attention"
    mixer: Any
    ff: Optional[int]                  # None: no feed-forward sublayer


def _need(ok: bool, what: str) -> None:
    if not ok:
        raise ValueError(f"Golitar config: {what}")


def _heads(m: Dict[str, Any], where: str):
    H, G, D, V = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    _need(G >= 1 and H >= 1 and H % G == 0, f"{where}: heads must be a multiple of kv_heads")
    _need(1 <= D <= 256 and 1 <= V <= 256, f"{where}: dim and vdim up to 256")
    return H, G, D, V


def _layer(d: Dict[str, Any], i: int) -> LayerConfig:
    where, m = f"layer {i}", d["mixer"]
    H, G, D, V = _heads(m, where)
    if d["type"] == "delta":
        _need(int(m["conv"]) >= 1, f"{where}: conv taps")
        mixer = DeltaMixerConfig(H, G, D, V, int(m["conv"]))
    elif d["type"] == "attention":
        r = m["rot"]
        dims = int(r["dims"])
        _need(dims % 2 == 0 and 0 <= dims <= D, f"{where}: rot.dims even and at most dim")
        sc = r.get("scaling")
        rot = RotaryConfig(dims, float(r["base"])) if not sc else RotaryConfig(
            dims, float(r["base"]), float(sc["factor"]), float(sc["low"]), float(sc["high"]), float(sc["original"]))
        mask = m.get("mask")
        window = int(mask["size"]) if mask else 0
        _need(not mask or window >= 1, f"{where}: mask.size")
        mixer = AttentionMixerConfig(H, G, D, V, float(m["diff"]), float(m["scale"]), rot,
                                     float(m.get("softcap") or 0.0), window)
    else:
        raise ValueError(f"Golitar config: {where}: unknown mixer type {d['type']!r}")
    mlp = d.get("mlp")
    if mlp is not None:
        _need(mlp.get("kind") == "dense", f"{where}: unknown feed-forward kind {mlp.get('kind')!r}")
    return LayerConfig(d["type"], mixer, int(mlp["ff"]) if mlp is not None else None)


class GolitarConfig:
    """Also carries the attribute names the inference application reads of every model configuration
    (hidden_size, vocab_size, num_attention_heads, rms_norm_eps, eos / pad token ids)."""

    model_type = "golitar"

    def __init__(self, raw: Dict[str, Any]):
        self.raw = copy.deepcopy(raw)
        name = raw.get("architecture", ARCHITECTURE)
        _need(name == ARCHITECTURE, f"architecture is {name!r}")
        self.layers: List[LayerConfig] = [_layer(d, i) for i, d in enumerate(raw["layers"])]
        self.vocab_size, self.hidden_size = int(raw["vocab"]), int(raw["width"])
        self.streams = int(raw["streams"])
        _need(1 <= self.streams <= 8, "1 to 8 streams")
        _need(1 <= self.hidden_size <= 16384, "width up to 16384")
        self.rms_norm_eps = float(raw["norm"]["eps"])
        self.logit_softcap = float(raw.get("logit_softcap") or 0.0)
        self.num_hidden_layers = len(self.layers)
        self.num_attention_heads = max((l.mixer.heads for l in self.layers), default=1)
        self.num_key_value_heads = max((l.mixer.kv_heads for l in self.layers), default=1)
        self.eos_token_id = raw.get("eos_token_id")
        self.pad_token_id = raw.get("pad_token_id")
        self.tie_word_embeddings = False

    @classmethod
    def from_pretrained(cls, path: str) -> "GolitarConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls(json.load(f))

    def save_pretrained(self, path: str) -> None:
        os.makedirs(path, exist_ok=True)
        with open(os.path.join(path, "config.json"), "w") as f:
            json.dump({"architecture": ARCHITECTURE, **self.raw}, f, indent=1)
