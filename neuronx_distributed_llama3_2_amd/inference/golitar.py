"""Golitar inference application and runner: the lifecycle of every model of the framework
(from_pretrained -> compile -> load -> generate; graph-captured token generation, bucketed context
encoding, on-device sampling) over the Golitar device module."""

from __future__ import annotations

from ..models.golitar import GolitarConfig, checkpoint_to_nxd
from .hybrid_app import HybridForCausalLMInference, HybridRunner
from .modeling_golitar import GolitarInferenceModel


class GolitarForCausalLMInference(HybridForCausalLMInference):
    _model_cls = GolitarInferenceModel

    @staticmethod
    def _hf_to_nxd(sd, model_config):
        return checkpoint_to_nxd(sd, model_config)

    @staticmethod
    def _config_from_dir(path: str):
        return GolitarConfig.from_pretrained(path)


class GolitarRunner(HybridRunner):
    app_cls = GolitarForCausalLMInference
