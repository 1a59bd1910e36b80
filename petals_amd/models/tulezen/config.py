"""Tulezen config: a decoder described layer by layer.

config.json gives ``vocab``, ``width``, ``norm.eps`` and a list ``layers``; each
entry names its mixer, the mixer's own sizes and constants, and its
feed-forward (or null). Nothing is uniform across layers: every size is read
from the entry, so blocks of one model may differ in heads, head sizes, latent
rank, window and experts.
"""

from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, FrozenSet, List, Optional, Tuple

import torch

from petals_amd.models.config_base import ModelConfig, register_config


@dataclasses.dataclass(frozen=True)
class LatentAttentionSpec:
    """Latent (MLA-style) attention without positions over a sliding window."""

    heads: int
    dim: int  # query/key dimensions per head
    vdim: int  # value dimensions per head
    kv_rank: int  # latent size; the only thing that is cached
    scale: float
    window: int  # position i sees j with 0 <= i - j < window; 0: all j <= i
    kv_from: Optional[int]  # layer whose cached latent is read (None: its own)


@dataclasses.dataclass(frozen=True)
class MoESpec:
    """Routed experts, weighted by their softmax score over all experts."""

    experts: int
    top: int
    ff: int
    limit: float  # clamp of the gated activation


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    attention: LatentAttentionSpec
    moe: Optional[MoESpec]


def _parse_layer(index: int, entry: Dict[str, Any]) -> LayerSpec:
    if entry.get("type") != "latent_attention":
        raise ValueError(f"layer {index}: unknown mixer type {entry.get('type')!r}")
    m = entry["mixer"]
    mask = m.get("mask") or {}
    attention = LatentAttentionSpec(
        heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
        scale=float(m["scale"]), window=int(mask.get("size", 0)),
        kv_from=None if m.get("kv_from") is None else int(m["kv_from"]),
    )
    if min(attention.heads, attention.dim, attention.vdim, attention.kv_rank) < 1 or attention.window < 0:
        raise ValueError(f"layer {index}: mixer sizes must be positive")
    moe = None
    f = entry.get("mlp")
    if f is not None:
        if f.get("kind", "moe") != "moe":
            raise ValueError(f"layer {index}: unknown feed-forward kind {f.get('kind')!r}")
        moe = MoESpec(
            experts=int(f["router"]["experts"]), top=int(f["router"]["top"]),
            ff=int(f["expert"]["ff"]), limit=float(f["expert"]["limit"]),
        )
        if not 1 <= moe.top <= moe.experts or moe.ff < 1:
            raise ValueError(f"layer {index}: {moe.top} of {moe.experts} experts of size {moe.ff}")
    return LayerSpec(attention, moe)


@register_config("tulezen", architecture="Tulezen")
@dataclasses.dataclass
class TulezenConfig(ModelConfig):
    layers: List[Dict[str, Any]] = dataclasses.field(default_factory=list)
    block_prefix: str = "l"

    kernel_library: ClassVar[str] = "latent"
    unsupported: ClassVar[FrozenSet[str]] = frozenset({"adapters", "quantization", "tensor parallelism"})

    def __post_init__(self):
        super().__post_init__()
        self._specs = tuple(_parse_layer(i, e) for i, e in enumerate(self.layers))
        for i, spec in enumerate(self._specs):
            src = spec.attention.kv_from
            if src is None:
                continue
            if not 0 <= src < i or self._specs[src].attention.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from {src} must be an earlier layer with a latent of its own")
            if self._specs[src].attention.kv_rank != spec.attention.kv_rank:
                raise ValueError(f"layer {i}: kv_rank differs from that of layer {src}")

    @classmethod
    def from_hf_dict(cls, d: Dict[str, Any], name_or_path: str = "") -> "TulezenConfig":
        layers = list(d["layers"])
        mixers = [e["mixer"] for e in layers]
        experts = [e["mlp"] for e in layers if e.get("mlp") is not None]
        flat = {
            "hidden_size": int(d.get("width", d.get("hidden_size", 0))),
            "vocab_size": int(d.get("vocab", d.get("vocab_size", 0))),
            "layer_norm_eps": float(d["norm"]["eps"] if "norm" in d else d["layer_norm_eps"]),
            "num_hidden_layers": len(layers),
            "num_attention_heads": max((int(m["heads"]) for m in mixers), default=1),
            "num_key_value_heads": 1,
            "intermediate_size": max((int(f["expert"]["ff"]) for f in experts), default=0),
            "max_position_embeddings": int(d.get("max_position_embeddings", 1 << 20)),
        }
        return super().from_hf_dict({**d, **flat}, name_or_path=name_or_path)

    def spec(self, block_index: int) -> LayerSpec:
        return self._specs[block_index]

    # ------------------------------------------- checkpoint and span layout

    def block_tensor_prefix(self, block_index: int) -> str:
        return f"{self.block_prefix}{block_index}."

    def client_tensor_names(self) -> Tuple[str, str, str]:
        return "embed", "final.norm", "head"

    def stream_dtype(self, dtype: torch.dtype) -> torch.dtype:
        return torch.float32  # the residual sum is kept in 32-bit

    def valid_cuts(self) -> Optional[FrozenSet[int]]:
        """A cut at c separates blocks < c from blocks >= c; none may fall
        between a layer and the layer whose latent it reads."""
        n = len(self._specs)
        cuts = set(range(n + 1))
        for i, spec in enumerate(self._specs):
            if spec.attention.kv_from is not None:
                cuts -= set(range(spec.attention.kv_from + 1, i + 1))
        return frozenset(cuts)

    def block_param_count(self) -> int:
        def count(s: LayerSpec) -> int:
            a, h = s.attention, self.hidden_size
            n = a.heads * a.dim * (h + a.kv_rank) + a.heads * a.vdim * (h + a.kv_rank)
            if a.kv_from is None:
                n += a.kv_rank * h
            if s.moe is not None:
                n += s.moe.experts * h * (3 * s.moe.ff + 1)
            return n

        return max((count(s) for s in self._specs), default=1)

    def cache_values_per_token(self, block_index: int = 0) -> int:
        a = self._specs[block_index].attention
        return 0 if a.kv_from is not None else -(-a.kv_rank // 32) * 32
