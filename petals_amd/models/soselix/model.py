"""Distributed Soselix model classes: client-side scaled embedding, final norm, head.

The hidden states that the client exchanges with the servers are the 32-bit
residual stream whatever the weight dtype is; the final norm runs in 32-bit and
only the head's product uses the weight dtype.
"""

from __future__ import annotations

import torch
from torch import nn

from petals_amd import ops
from petals_amd.models.model_base import (
    DistributedForCausalLMBase,
    DistributedForSequenceClassificationBase,
    DistributedModelBase,
)


class _SingleWeightNorm(nn.Module):
    """RMS norm with one weight for all coordinates, 32-bit in and out."""

    def __init__(self, eps: float):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(()))
        self.eps = eps

    def forward(self, x):
        return ops.rms_norm_f32(x.float(), self.weight.expand(x.shape[-1]), self.eps)


class DistributedSoselixModel(DistributedModelBase):
    def _make_final_norm(self, config):
        return _SingleWeightNorm(config.layer_norm_eps)

    def _prepare_embeds(self, inputs_embeds: torch.Tensor) -> torch.Tensor:
        return inputs_embeds.float() * self.config.embedding_scale

    @property
    def layers(self):
        return self.h


class DistributedSoselixForCausalLM(DistributedForCausalLMBase):
    @classmethod
    def _build(cls, config):
        return cls(config, model=DistributedSoselixModel(config))


class DistributedSoselixForSequenceClassification(DistributedForSequenceClassificationBase):
    @classmethod
    def from_pretrained(cls, model_name_or_path: str, config=None, num_labels: int = 2, **kwargs):
        if config is None:
            from petals_amd.utils.auto_config import AutoDistributedConfig

            config = AutoDistributedConfig.from_pretrained(model_name_or_path, **kwargs)
        return cls(config, model=DistributedSoselixModel(config), num_labels=num_labels)
