"""Bezurax model configuration: the reader of its config.json.

A Bezurax decoder is a list of layers; each has two mixers side by side on the same normalised input
(left: attention over a window and pooled blocks, right: a delta rule with decay and removal per
channel) and, parallel to them, a mixture-of-experts feed-forward or none.  A layer may use the weights
of another one.  The width of the decay's low-rank projection is a tensor's shape: it is read from the
checkpoint's header, and kept under "rank" when the configuration is saved."""

from __future__ import annotations

import copy
import json
import os
import struct
from dataclasses import dataclass
from typing import Any, Dict, List, Optional

ARCHITECTURE = "Bezurax"


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: int
    pool: int


@dataclass(frozen=True)
class DeltaConfig:
    heads: int
    dim: int
    rank: int


@dataclass(frozen=True)
class ParallelMixerConfig:
    left: AttentionConfig
    right: DeltaConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class ExpertsConfig:
    experts: int
    top: int
    ff: int
    limit: float
    scale: float
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0          # 0: no shared expert
    shared_limit: float = 0.0


@dataclass(frozen=True)
class LayerConfig:
    mixer: ParallelMixerConfig
    mlp: Optional[ExpertsConfig]
    weights: int                # the layer of this list whose weights it uses (itself, usually)


def _need(ok: bool, what: str) -> None:
    if not ok:
        raise ValueError(f"Bezurax config: {what}")


def tensor_shapes(path: str) -> Dict[str, List[int]]:
    """Shapes of every tensor of a safetensors checkpoint directory, from the files' headers."""
    out: Dict[str, List[int]] = {}
    for name in sorted(os.listdir(path)):
        if not name.endswith(".safetensors"):
            continue
        with open(os.path.join(path, name), "rb") as f:
            n = struct.unpack("<Q", f.read(8))[0]
            out.update({k: v["shape"] for k, v in json.loads(f.read(n)).items() if k != "__metadata__"})
    return out


def _mixer(m: Dict[str, Any], where: str) -> ParallelMixerConfig:
    a, d = m["left"], m["right"]
    H, G, D = int(a["heads"]), int(a["kv_heads"]), int(a["dim"])
    _need(G >= 1 and H >= 1 and H % G == 0, f"{where}: heads must be a multiple of kv_heads")
    _need(2 <= D <= 256, f"{where}: dim up to 256")
    _need(int(a.get("vdim", D)) == D, f"{where}: values are the keys, vdim must equal dim")
    window, pool = int(a["mask"]["size"]), int(a["mask"]["pool"])
    _need(window >= 1 and pool >= 1, f"{where}: mask.size and mask.pool")
    R, E, rank = int(d["heads"]), int(d["dim"]), int(d.get("rank", 0))
    _need(R >= 1 and 1 <= E <= 256, f"{where}: right heads and dim (up to 256)")
    _need(rank >= 1, f"{where}: the rank of the decay's projection is missing")
    return ParallelMixerConfig(AttentionConfig(H, G, D, float(a["scale"]), window, pool), DeltaConfig(R, E, rank),
                               float(m["left_scale"]), float(m["right_scale"]))


def _experts(m: Dict[str, Any], where: str) -> ExpertsConfig:
    _need(m.get("kind") == "moe", f"{where}: unknown feed-forward kind {m.get('kind')!r}")
    r, e, s = m["router"], m["expert"], m.get("shared")
    n, top = int(r["experts"]), int(r["top"])
    g = r.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(g["count"]), int(g["keep"])
    _need(1 <= n <= 1024 and count >= 1 and n % count == 0 and 1 <= keep <= count, f"{where}: expert groups")
    _need(1 <= top <= keep * (n // count), f"{where}: router.top")
    return ExpertsConfig(n, top, int(e["ff"]), float(e["limit"]), float(r["scale"]), count, keep,
                         int(s["ff"]) if s else 0, float(s["limit"]) if s else 0.0)


class BezuraxConfig:
    """Also carries the attribute names the inference application reads of every model configuration
    (hidden_size, vocab_size, num_attention_heads, rms_norm_eps, eos / pad token ids)."""

    model_type = "bezurax"

    def __init__(self, raw: Dict[str, Any]):
        self.raw = copy.deepcopy(raw)
        name = raw.get("architecture", ARCHITECTURE)
        _need(name == ARCHITECTURE, f"architecture is {name!r}")
        self.vocab_size, self.hidden_size = int(raw["vocab"]), int(raw["width"])
        _need(1 <= self.hidden_size <= 16384, "width up to 16384")
        self.rms_norm_eps = float(raw["norm"]["eps"])
        self.norm_groups = int(raw["norm"]["groups"])
        _need(self.norm_groups >= 1 and self.hidden_size % self.norm_groups == 0, "norm.groups must divide the width")
        self.layers: List[LayerConfig] = []
        for i, d in enumerate(raw["layers"]):
            where = f"layer {i}"
            if d["type"] != "parallel":
                raise ValueError(f"Bezurax config: {where}: unknown mixer type {d['type']!r}")
            self.layers.append(LayerConfig(_mixer(d["mixer"], where), _experts(d["mlp"], where) if d.get("mlp") else None,
                                           owner(raw["layers"], i)))
        for i, layer in enumerate(self.layers):
            own = self.layers[layer.weights]
            _need((own.mixer, own.mlp) == (layer.mixer, layer.mlp), f"layer {i} differs from the layer whose weights it uses")
        # layers that have weights, in order; layer i runs with weights unique[use[i]]
        self.unique = [i for i, layer in enumerate(self.layers) if layer.weights == i]
        self.use = [self.unique.index(layer.weights) for layer in self.layers]
        self.logit_scale = float(raw["logit_scale"])
        self.num_hidden_layers = len(self.layers)
        self.num_attention_heads = max((l.mixer.left.heads for l in self.layers), default=1)
        self.num_key_value_heads = max((l.mixer.left.kv_heads for l in self.layers), default=1)
        self.eos_token_id = raw.get("eos_token_id")
        self.pad_token_id = raw.get("pad_token_id")
        self.tie_word_embeddings = True

    @classmethod
    def from_pretrained(cls, path: str) -> "BezuraxConfig":
        with open(os.path.join(path, "config.json")) as f:
            raw = json.load(f)
        missing = [i for i, d in enumerate(raw["layers"]) if "rank" not in d["mixer"].get("right", {"rank": 0})]
        if missing:
            shapes = tensor_shapes(path)
            for i in missing:
                name = f"l{owner(raw['layers'], i)}.mix.right.w1"
                if name in shapes:
                    raw["layers"][i]["mixer"]["right"]["rank"] = shapes[name][0]
        return cls(raw)

    def save_pretrained(self, path: str) -> None:
        os.makedirs(path, exist_ok=True)
        with open(os.path.join(path, "config.json"), "w") as f:
            json.dump({"architecture": ARCHITECTURE, **self.raw}, f, indent=1)


def owner(layers, i: int) -> int:
    """The layer whose weights layer i uses."""
    seen = [i]
    while layers[i].get("weights_of") is not None:
        i = int(layers[i]["weights_of"])
        _need(0 <= i < len(layers) and i not in seen, f"layer {seen[0]}: weights_of")
        seen.append(i)
    return i
