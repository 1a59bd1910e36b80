"""Distributed Zudarax model classes: client-side embedding, final norm, head.

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


class _GroupedNorm(nn.Module):
    """RMS norm in equal parts, 32-bit in and out."""

    def __init__(self, hidden_size: int, groups: int, eps: float):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(hidden_size))
        self.groups, self.eps = groups, eps

    def forward(self, x):
        return ops.rms_norm_f32(x.float(), self.weight, self.eps, self.groups)


class DistributedZudaraxModel(DistributedModelBase):
    def _make_final_norm(self, config):
        return _GroupedNorm(config.hidden_size, config.norm_groups, config.layer_norm_eps)

    def _prepare_embeds(self, inputs_embeds: torch.Tensor) -> torch.Tensor:
        return inputs_embeds.float()

    @property
    def layers(self):
        return self.h


class DistributedZudaraxForCausalLM(DistributedForCausalLMBase):
    @classmethod
    def _build(cls, config):
        return cls(config, model=DistributedZudaraxModel(config))


class DistributedZudaraxForSequenceClassification(DistributedForSequenceClassificationBase):
    @classmethod
    def from_pretrained(cls, model_name_or_path: str, config=None, num_labels: int = 2, **kwargs):
        if config is None:
            from petals_amd.utils.auto_config import AutoDistributedConfig

            config = AutoDistributedConfig.from_pretrained(model_name_or_path, **kwargs)
        return cls(config, model=DistributedZudaraxModel(config), num_labels=num_labels)
