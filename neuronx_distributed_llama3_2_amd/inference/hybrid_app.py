"""What the applications and runners of hybrid decoders share: no int8 weights, no speculation over a
recurrent state, accuracy checked against the same model in 32-bit."""

from __future__ import annotations

from typing import Optional, Sequence

import torch

from .generation import LlamaForCausalLMInference
from .runner import InferenceRunner


class HybridForCausalLMInference(LlamaForCausalLMInference):
    def _quantize(self) -> None:
        raise NotImplementedError("int8 weight-only quantization is implemented for dense decoders only")

    def generate(self, input_ids, attention_mask=None, **kwargs):
        if kwargs.get("assistant_model") is not None:
            raise NotImplementedError("speculative decoding needs a cache that can step back; a recurrent state cannot")
        return super().generate(input_ids, attention_mask, **kwargs)


class HybridRunner(InferenceRunner):
    def load_hf_model(self):
        raise NotImplementedError("no library implements this design")

    def generate_with_hf(self, prompts: Sequence, max_length: int, **kwargs):
        raise NotImplementedError("no library implements this design")

    def check_accuracy(self, model, prompts: Sequence, max_length: Optional[int] = None,
                       num_tokens_to_check: Optional[int] = None) -> bool:
        """Greedy tokens of `model` == the same model computed in 32-bit, one sequence at a time."""
        max_length = max_length or model.config.max_length
        ids, mask = self._encode(prompts)
        got = model.generate(ids, mask, max_new_tokens=max_length - ids.shape[1], eos_token_id=None).cpu()
        ref = self.load_neuron_model_on_cpu(ids.shape[1], max_length, 1)
        ok = True
        for i in range(ids.shape[0]):
            n = int(mask[i].sum())
            want = ref.generate(ids[i:i + 1, :n], max_new_tokens=max_length - ids.shape[1], eos_token_id=None).cpu()[0, n:]
            k = num_tokens_to_check or want.numel()
            ok = ok and torch.equal(want[:k], got[i, ids.shape[1]:ids.shape[1] + k])
        return ok
