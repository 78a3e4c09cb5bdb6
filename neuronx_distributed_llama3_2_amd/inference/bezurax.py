"""Bezurax inference application and runner: the lifecycle of every model of the framework
(from_pretrained -> compile -> load -> generate; graph-captured token generation, bucketed context
encoding, on-device sampling) over the Bezurax device module."""

from __future__ import annotations

from ..models.bezurax import BezuraxConfig, checkpoint_to_nxd
from .hybrid_app import HybridForCausalLMInference, HybridRunner
from .modeling_bezurax import BezuraxInferenceModel


class BezuraxForCausalLMInference(HybridForCausalLMInference):
    _model_cls = BezuraxInferenceModel

    @staticmethod
    def _hf_to_nxd(sd, model_config):
        return checkpoint_to_nxd(sd, model_config)

    @staticmethod
    def _config_from_dir(path: str):
        return BezuraxConfig.from_pretrained(path)


class BezuraxRunner(HybridRunner):
    app_cls = BezuraxForCausalLMInference
