"""Golitar inference model: hyper-connected residual streams around gated-delta-rule and differential-
attention mixers and squared-ReLU feed-forwards.

The residual is [rows, streams, width] in fp32; between two sublayers one kernel (ops.hyper_step)
writes the last sublayer's output into the streams and reads and normalises the next one's input, so a
layer of the forward is: hyper_step, projection GEMM, mixer kernels, output GEMM (and the same around the
feed-forward).  A decode step of up to 4 sequences folds the norms into the input projections and the
stream updates into the output projections (_forward_decode_fused_streams).  The step function, cache set-up and decode-graph hooks are those of every
model of the framework (model_base.DecoderInferenceMixin); the cache is a LayerCache.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..models.golitar import GolitarConfig
from ..modules.hybrid import (DifferentialAttentionMixer, GatedDeltaMixer, HyperConnection, SquaredReluMLP,
                              StepContext)
from ..modules.hybrid.context import small
from ..ops.gemm import linear_f32
from ..ops.hyper import FUSED_NORM_ELEMENTS, FUSED_ROWS
from ..parallel_layers.parallel_state import get_tensor_model_parallel_size
from .layer_cache import LayerCache
from .model_base import DecoderInferenceMixin


class GolitarLayer(nn.Module):
    def __init__(self, cfg, config: GolitarConfig, dtype, device):
        super().__init__()
        W, eps, m = config.hidden_size, config.rms_norm_eps, cfg.mixer
        if cfg.type == "delta":
            self.mixer = GatedDeltaMixer(W, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, eps, dtype, device)
        else:
            self.mixer = DifferentialAttentionMixer(W, m.heads, m.kv_heads, m.dim, m.vdim, m.diff, m.scale, m.rot, eps,
                                                    m.softcap, m.window, dtype, device)
        self.mlp = SquaredReluMLP(W, cfg.ff, dtype, device) if cfg.ff is not None else None
        n = 1 if cfg.ff is None else 2   # sublayers
        self.norms = nn.ParameterList([small(W, device=device) for _ in range(n)])
        self.hyper = nn.ModuleList([HyperConnection(config.streams, device) for _ in range(n)])


class GolitarModel(nn.Module):
    def __init__(self, config: GolitarConfig, dtype, device):
        super().__init__()
        self.embed_tokens = nn.Embedding(config.vocab_size, config.hidden_size, dtype=dtype, device=device)
        self.layers = nn.ModuleList([GolitarLayer(c, config, dtype, device) for c in config.layers])
        self.norm = nn.Module()
        self.norm.weight = small(config.hidden_size, device=device)


class GolitarInferenceModel(DecoderInferenceMixin, nn.Module):
    def __init__(self, config: GolitarConfig, dtype=torch.bfloat16, device=None):
        nn.Module.__init__(self)
        if get_tensor_model_parallel_size() != 1:
            raise NotImplementedError("Golitar runs on one GPU (tensor parallel degree 1)")
        self.config = config
        self.model = GolitarModel(config, dtype, device)
        self.lm_head = nn.Linear(config.hidden_size, config.vocab_size, bias=False, dtype=dtype, device=device)
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
        self.model.norm.weight.zero_()
        for layer in self.model.layers:
            layer.mixer.reset_parameters()
            for n, hc in zip(layer.norms, layer.hyper):
                n.zero_()
                hc.reset_parameters()

    def post_load(self) -> None:
        for layer in self.model.layers:
            if hasattr(layer.mixer, "weights_changed"):
                layer.mixer.weights_changed()
        if self._decode_fused_ok:   # (kept off when it was switched off)
            self._decode_fused_ok = None

    # ------------------------------------------------------------------ cache
    def setup_kv_cache(self, max_batch: int, max_len: int, device=None) -> LayerCache:
        emb = self.model.embed_tokens.weight
        device = device or emb.device
        mixers = [layer.mixer for layer in self.model.layers]
        if self.kv_cache is None or not self.kv_cache.matches(max_batch, max_len, emb.dtype, device):
            self.kv_cache = None   # release before the new one is allocated
            self.kv_cache = LayerCache(mixers, max_batch, max_len, emb.dtype, device)
        for m in mixers:
            if hasattr(m, "prepare"):
                m.prepare(max_len, device)
        return self.kv_cache

    def save_cache(self):
        return self.kv_cache.save()

    def load_cache(self, saved) -> None:
        self.kv_cache.load(saved)

    # ------------------------------------------------------------------ forward
    def _sublayers(self):
        """(cache index, module, hyper-connection, norm) of every sublayer in order."""
        for i, layer in enumerate(self.model.layers):
            yield i, layer.mixer, layer.hyper[0], layer.norms[0]
            if layer.mlp is not None:
                yield None, layer.mlp, layer.hyper[1], layer.norms[1]

    def _fused(self, input_ids: torch.Tensor) -> bool:
        """Fused kernels wanted (set_fused_decode) and possible (GPU)."""
        return self._decode_fused_ok is not False and input_ids.is_cuda

    def _check_decode_fusable(self) -> bool:
        ws = [self.lm_head.weight] + [m.weight for _, mod, _, _ in self._sublayers() for m in (mod.in_linear, mod.out_linear)]
        return all(w.dtype == torch.bfloat16 and w.shape[1] % 8 == 0 and w.is_contiguous() for w in ws)

    def _decode_fusable(self, input_ids: torch.Tensor) -> bool:
        """One new token for up to FUSED_ROWS sequences with every projection a fused GEMV."""
        if not self._fused(input_ids):
            return False
        if self._decode_fused_ok is None:
            self._gemv_ok = self._check_decode_fusable()
            self._decode_fused_ok = True
        M = input_ids.shape[0]
        return (self._gemv_ok and input_ids.shape[1] == 1 and M <= FUSED_ROWS
                and M * self.config.hidden_size <= FUSED_NORM_ELEMENTS)

    @torch.no_grad()
    def forward_tokens(self, input_ids: torch.Tensor, positions: torch.Tensor, seq_ids: Optional[torch.Tensor] = None,
                       cache_len: Optional[torch.Tensor] = None, last_index: Optional[torch.Tensor] = None,
                       prefill: bool = False, return_hidden: bool = False, lengths: Optional[torch.Tensor] = None,
                       logit_rows: Optional[torch.Tensor] = None):
        """As DecoderInferenceMixin.forward_tokens; logits are fp32."""
        assert self.kv_cache is not None, "call setup_kv_cache() first"
        B, T = input_ids.shape
        step = self.kv_cache.max_step
        if not prefill and T > step:   # more new tokens than the windowed rings take at once
            return self._forward_in_steps(input_ids, positions, seq_ids, last_index, return_hidden, lengths, logit_rows,
                                          step)
        if lengths is None and last_index is not None and prefill:
            lengths = last_index + 1
        ctx = StepContext(B, T, positions if positions.dtype == torch.int64 else positions.long(),
                          lengths.to(torch.int32) if lengths is not None else None,
                          seq_ids.to(torch.int32) if seq_ids is not None else None, prefill,
                          self._fused(input_ids))
        emb = self.model.embed_tokens.weight
        M, dt = B * T, emb.dtype
        if logit_rows is None and last_index is not None:
            logit_rows = torch.arange(B, device=input_ids.device) * T + last_index
        streams = torch.empty((M, self.config.streams, emb.shape[1]), dtype=torch.float32, device=emb.device)
        last = dict(embed=emb, ids=input_ids.reshape(-1).to(torch.int64).contiguous())
        if not prefill and lengths is None and self._decode_fusable(input_ids):
            return self._forward_decode_fused_streams(streams, last, ctx, logit_rows, return_hidden)
        for index, mod, hc, norm in self._sublayers():
            h = ops.hyper_step(streams, read=hc.read, norm_w=norm, eps=self.eps, dtype=dt, **last)
            y = mod(h, self.kv_cache[index] if index is not None else None, ctx)
            last = dict(y=y, y_bias=mod.o_bias, mix=hc.mix, write=hc.write)
        h = ops.hyper_step(streams, read=self._ones(emb.device), norm_w=self.model.norm.weight, eps=self.eps, dtype=dt,
                           rows=logit_rows, store=False, **last)
        logits = self._logits(h)
        if logit_rows is None:
            logits, h = logits.view(B, T, -1), h.view(B, T, -1)
        return (logits, h) if return_hidden else logits

    def _forward_decode_fused_streams(self, streams, start, ctx, logit_rows, return_hidden):
        """One new token per sequence.  A sublayer is three launches: norm + input projection, mixer core
        (none for a feed-forward), output projection + streams; the first one's input comes from the
        embedding launch, the last streams launch reads their sum for the final norm + lm_head."""
        subs = list(self._sublayers())
        ones = self._ones(streams.device)
        dt = self.model.embed_tokens.weight.dtype
        x, u = ops.hyper_step(streams, read=subs[0][2].read, norm_w=subs[0][3], eps=self.eps, dtype=dt, **start), None
        for i, (index, mod, hc, norm) in enumerate(subs):
            a = ops.decode_linear(mod.in_linear.weight, x, u, None if u is None else norm, self.eps, mod.in_epilogue)
            a = mod.core(a, self.kv_cache[index] if index is not None else None, ctx)
            read = subs[i + 1][2].read if i + 1 < len(subs) else ones
            u = ops.decode_linear_into_streams(mod.out_linear.weight, a, streams, mod.o_bias, hc.mix, hc.write, read)
            x = None
        norm = self.model.norm.weight
        if logit_rows is not None:
            u = u[logit_rows]
        logits = ops.decode_linear(self.lm_head.weight, None, u, norm, self.eps, "f32", self.config.logit_softcap)
        if not return_hidden:
            return logits if logit_rows is not None else logits.unsqueeze(1)
        h = (u * torch.rsqrt(u.square().mean(-1, keepdim=True) + self.eps) * (1 + norm)).to(dt)
        return (logits, h) if logit_rows is not None else (logits.unsqueeze(1), h.unsqueeze(1))

    def _ones(self, device) -> torch.Tensor:
        if getattr(self, "_ones_buf", None) is None or self._ones_buf.device != device:
            self._ones_buf = torch.ones(self.config.streams, dtype=torch.float32, device=device)
        return self._ones_buf

    def _logits(self, h: torch.Tensor) -> torch.Tensor:
        logits = linear_f32(h, self.lm_head.weight)
        return ops.softcap_(logits, self.config.logit_softcap) if self.config.logit_softcap > 0 else logits

    def forward_tree(self, *a, **k):
        raise NotImplementedError("tree verification needs a cache without a recurrent state")
