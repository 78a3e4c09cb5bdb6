"""Bezurax inference model: layers whose mixers (attention with pooled blocks beside a generalised delta
rule) and routed experts read the same fp32 residual.

Between two layers one kernel (ops.residual_norms) adds everything the last layer brought to the residual
and normalises it twice.  Layers may share weights: `model.layers` holds those that have some, the
configuration's `use` names the one each layer runs with; every layer has a cache of its own.  The step
function, cache set-up and decode-graph hooks are those of every model of the framework
(model_base.DecoderInferenceMixin); the cache is a LayerCache.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..models.bezurax import BezuraxConfig
from ..modules.hybrid import ChannelDelta, ParallelMixer, PooledAttention, RoutedExperts, StepContext
from ..modules.hybrid.context import few_rows, small
from ..ops.experts import RouterRule
from ..ops.gemm import linear_f32
from ..parallel_layers.parallel_state import get_tensor_model_parallel_size
from .layer_cache import LayerCache
from .model_base import DecoderInferenceMixin


class BezuraxLayer(nn.Module):
    def __init__(self, cfg, config: BezuraxConfig, dtype, device):
        super().__init__()
        W, eps, a, d, e = config.hidden_size, config.rms_norm_eps, cfg.mixer.left, cfg.mixer.right, cfg.mlp
        self.mixer = ParallelMixer(W, PooledAttention(a.heads, a.kv_heads, a.dim, a.scale, a.window, a.pool, eps, device),
                                   ChannelDelta(d.heads, d.dim, d.rank, eps, dtype, device), cfg.mixer.left_scale,
                                   cfg.mixer.right_scale, dtype, device)
        self.mlp = None
        if e is not None:
            self.mlp = RoutedExperts(W, RouterRule(e.experts, e.top, e.scale, e.groups, e.keep), e.ff, e.limit, e.shared_ff,
                                     e.shared_limit, dtype, device)
        self.norms = nn.ParameterList([small(W, device=device) for _ in range(1 if e is None else 2)])


class BezuraxModel(nn.Module):
    def __init__(self, config: BezuraxConfig, dtype, device):
        super().__init__()
        self.embed_tokens = nn.Embedding(config.vocab_size, config.hidden_size, dtype=dtype, device=device)
        self.layers = nn.ModuleList([BezuraxLayer(config.layers[i], config, dtype, device) for i in config.unique])
        self.norm = nn.Module()
        self.norm.weight = small(config.hidden_size, device=device)


class BezuraxInferenceModel(DecoderInferenceMixin, nn.Module):
    def __init__(self, config: BezuraxConfig, dtype=torch.bfloat16, device=None):
        nn.Module.__init__(self)
        if get_tensor_model_parallel_size() != 1:
            raise NotImplementedError("Bezurax runs on one GPU (tensor parallel degree 1)")
        self.config = config
        self.model = BezuraxModel(config, dtype, device)
        self.lm_head = nn.Linear(config.hidden_size, config.vocab_size, bias=False, dtype=dtype, device=device)
        self.lm_head.weight = self.model.embed_tokens.weight
        self.tp = 1
        self.eps = config.rms_norm_eps
        self.kv_cache: Optional[LayerCache] = None
        self._decode_fused_ok: Optional[bool] = None
        self.eval()
        for p in self.parameters():
            p.requires_grad_(False)
        if next(self.parameters()).device.type != "meta":
            self.reset_parameters()

    @torch.no_grad()
    def reset_parameters(self) -> None:
        """Random initialisation of what torch's modules leave empty."""
        self.model.norm.weight.fill_(1.0)
        for layer in self.model.layers:
            layer.mixer.reset_parameters()
            if layer.mlp is not None:
                layer.mlp.reset_parameters()
            for n in layer.norms:
                n.fill_(1.0)

    def post_load(self) -> None:
        if self._decode_fused_ok:   # (kept off when it was switched off)
            self._decode_fused_ok = None

    # ------------------------------------------------------------------ cache
    def runs(self):
        """The layers in the order they run, each with its index (of its cache)."""
        return [(i, self.model.layers[u]) for i, u in enumerate(self.config.use)]

    def setup_kv_cache(self, max_batch: int, max_len: int, device=None) -> LayerCache:
        emb = self.model.embed_tokens.weight
        device = device or emb.device
        if self.kv_cache is None or not self.kv_cache.matches(max_batch, max_len, emb.dtype, device):
            self.kv_cache = None   # release before the new one is allocated
            self.kv_cache = LayerCache([layer.mixer for _, layer in self.runs()], max_batch, max_len, emb.dtype, device)
        return self.kv_cache

    def save_cache(self):
        return self.kv_cache.save()

    def load_cache(self, saved) -> None:
        self.kv_cache.load(saved)

    # ------------------------------------------------------------------ forward
    @torch.no_grad()
    def forward_tokens(self, input_ids: torch.Tensor, positions: torch.Tensor, seq_ids: Optional[torch.Tensor] = None,
                       cache_len: Optional[torch.Tensor] = None, last_index: Optional[torch.Tensor] = None,
                       prefill: bool = False, return_hidden: bool = False, lengths: Optional[torch.Tensor] = None,
                       logit_rows: Optional[torch.Tensor] = None):
        """As DecoderInferenceMixin.forward_tokens; logits are fp32."""
        assert self.kv_cache is not None, "call setup_kv_cache() first"
        B, T = input_ids.shape
        if not prefill and T > self.kv_cache.max_step:   # more new tokens than the rings take at once
            return self._forward_in_steps(input_ids, positions, seq_ids, last_index, return_hidden, lengths, logit_rows,
                                          self.kv_cache.max_step)
        if lengths is None and last_index is not None and prefill:
            lengths = last_index + 1
        ctx = StepContext(B, T, positions if positions.dtype == torch.int64 else positions.long(),
                          lengths.to(torch.int32) if lengths is not None else None,
                          seq_ids.to(torch.int32) if seq_ids is not None else None, prefill,
                          self._decode_fused_ok is not False and input_ids.is_cuda)
        emb = self.model.embed_tokens.weight
        if logit_rows is None and last_index is not None:
            logit_rows = torch.arange(B, device=input_ids.device) * T + last_index
        x = torch.empty((B * T, emb.shape[1]), dtype=torch.float32, device=emb.device)
        last = dict(embed=emb, ids=input_ids.reshape(-1).to(torch.int64).contiguous())
        norm = dict(eps=self.eps, groups=self.config.norm_groups, dtype=emb.dtype)
        for i, layer in self.runs():
            hs = ops.residual_norms(x, list(layer.norms), **norm, **last)
            y = layer.mixer(hs[0], self.kv_cache[i], ctx)
            last = dict(adds=[y])
            if layer.mlp is not None:
                m = layer.mlp(hs[1], ctx.fused)
                last = dict(m, adds=[y, *m["adds"]])
        h = ops.residual_norms(x, [self.model.norm.weight], rows=logit_rows, store=False, **norm, **last)[0]
        w, scale = self.lm_head.weight, self.config.logit_scale
        if ctx.fused and few_rows(h, w):
            logits = ops.decode_linear(w, h, epilogue="f32", alpha=scale)
        else:
            logits = linear_f32(h, w, scale)
        if logit_rows is None:
            logits, h = logits.view(B, T, -1), h.view(B, T, -1)
        return (logits, h) if return_hidden else logits

    def forward_tree(self, *a, **k):
        raise NotImplementedError("tree verification needs a cache without a recurrent state")
