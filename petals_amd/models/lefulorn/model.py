"""Distributed Lefulorn model classes: client-side embedding, final norm, head.

The hidden states that the client exchanges with the servers are the 32-bit
residual stream, with room for the values that later layers mix in; the final
norm runs in 32-bit and only the head's product uses the weight dtype.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from petals_amd import ops
from petals_amd.models.model_base import (
    DistributedForCausalLMBase,
    DistributedForSequenceClassificationBase,
    DistributedModelBase,
)


class _StreamNorm(nn.Module):
    """RMS norm of the residual part of the stream, 32-bit in and out."""

    def __init__(self, hidden_size: int, eps: float):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(hidden_size))
        self.eps = eps

    def forward(self, x):
        return ops.rms_norm_f32(x[..., : self.weight.shape[0]].float(), self.weight, self.eps)


class DistributedLefulornModel(DistributedModelBase):
    def _make_final_norm(self, config):
        return _StreamNorm(config.hidden_size, config.layer_norm_eps)

    def _prepare_embeds(self, inputs_embeds: torch.Tensor) -> torch.Tensor:
        return F.pad(inputs_embeds.float(), (0, self.config.stream_width - inputs_embeds.shape[-1]))

    @property
    def layers(self):
        return self.h


class DistributedLefulornForCausalLM(DistributedForCausalLMBase):
    @classmethod
    def _build(cls, config):
        return cls(config, model=DistributedLefulornModel(config))


class DistributedLefulornForSequenceClassification(DistributedForSequenceClassificationBase):
    @classmethod
    def from_pretrained(cls, model_name_or_path: str, config=None, num_labels: int = 2, **kwargs):
        if config is None:
            from petals_amd.utils.auto_config import AutoDistributedConfig

            config = AutoDistributedConfig.from_pretrained(model_name_or_path, **kwargs)
        return cls(config, model=DistributedLefulornModel(config), num_labels=num_labels)
