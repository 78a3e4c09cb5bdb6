"""Model families by the name in a model directory's config.json: its inference application and its
runner.  `app_class(path)` is what every entry point that gets a directory uses (runner, SPMD workers,
trace replay)."""

from __future__ import annotations

import importlib
import json
import os
from typing import Dict, NamedTuple, Optional


class Family(NamedTuple):
    module: str        # of this package
    app: str
    runner: Optional[str]
    extension: str = "_C"   # the extension module its kernels are in (_build.TARGETS)


FAMILIES: Dict[str, Family] = {
    "llama": Family(".generation", "LlamaForCausalLMInference", None),
    "mixtral": Family(".moe", "MixtralForCausalLMInference", "MixtralRunner"),
    "dbrx": Family(".moe", "DbrxForCausalLMInference", "DbrxRunner"),
    "golitar": Family(".golitar", "GolitarForCausalLMInference", "GolitarRunner", "_hybrid"),
    "bezurax": Family(".bezurax", "BezuraxForCausalLMInference", "BezuraxRunner", "_hybrid"),
}


def register_family(name: str, family: Family) -> None:
    FAMILIES[name.lower()] = family


def family_name(config: dict) -> str:
    """Family of a parsed config.json: its architecture, architectures or model_type."""
    names = [config.get("architecture"), *(config.get("architectures") or []), config.get("model_type")]
    for n in filter(None, names):
        low = str(n).lower()
        for key in (low, low.replace("forcausallm", "")):
            if key in FAMILIES:
                return key
    raise ValueError(f"no model family for config.json with {[n for n in names if n]}; known: {sorted(FAMILIES)}")


def family_of(path: str) -> str:
    with open(os.path.join(path, "config.json")) as f:
        return family_name(json.load(f))


def app_class(path: str):
    """Inference application class of a model directory (or of a compiled one)."""
    fam = FAMILIES[family_of(path)]
    return getattr(importlib.import_module(fam.module, __package__), fam.app)


def extension_of(path: str) -> str:
    return FAMILIES[family_of(path)].extension


def runner_class(path: str):
    fam = FAMILIES[family_of(path)]
    if fam.runner is None:
        from .runner import LlamaRunner

        return LlamaRunner
    return getattr(importlib.import_module(fam.module, __package__), fam.runner)
