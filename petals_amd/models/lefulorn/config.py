"""Lefulorn config: pre-norm decoder layers that mix tokens with a gated delta
rule or with windowed attention, described layer by layer.

config.json gives ``vocab``, ``width``, ``norm.eps``, ``logit_scale`` and a list
``layers``; each entry names its mixer (``type``), the mixer's own sizes and
constants, and its feed-forward (or null). Nothing is uniform across layers. The
ranks of the low-rank projections are given by the checkpoint's tensors.
"""

from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, FrozenSet, List, Optional, Tuple, Union

import torch

from petals_amd.models.config_base import ModelConfig, register_config

KEY_PAD, VALUE_PAD = 32, 16  # head sizes in the cache are rounded up to these (ops/hybrid.py)


@dataclasses.dataclass(frozen=True)
class DeltaSpec:
    """Gated delta rule with one decay per head and key channel."""

    heads: int
    kv_heads: int  # query/key heads
    dim: int  # query/key dimensions per head
    vdim: int  # value dimensions per head
    taps: int  # short convolution, the current token included


@dataclasses.dataclass(frozen=True)
class AttentionSpec:
    """Sliding-window attention with a distance bias, a sink and an output gate."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int  # position i sees j with 0 <= i - j < window; 0: all j <= i
    temp_coef: float  # query factor 1 + coef * ln(floor((p + 1) / every) + 1)
    temp_every: int
    v_mix: bool  # values are mixed with those of the first such layer


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    ff: int


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: Union[DeltaSpec, AttentionSpec]
    mlp: Optional[DenseSpec]


def _whole(value) -> int:
    if int(value) != value:
        raise ValueError(f"{value!r} is not a whole number")
    return int(value)


def _parse_layer(index: int, entry: Dict[str, Any]) -> LayerSpec:
    kind, m = entry.get("type"), entry["mixer"]
    sizes = dict(
        heads=_whole(m["heads"]), kv_heads=_whole(m.get("kv_heads", m["heads"])), dim=_whole(m["dim"]),
        vdim=_whole(m["vdim"]),
    )
    if min(sizes.values()) < 1 or sizes["heads"] % sizes["kv_heads"]:
        raise ValueError(f"layer {index}: mixer sizes {sizes}")
    if kind == "channel_delta":
        mixer = DeltaSpec(**sizes, taps=_whole(m["conv"]))
        if mixer.taps < 1:
            raise ValueError(f"layer {index}: a convolution of {mixer.taps} taps")
    elif kind == "attention":
        temp = m.get("q_temp") or {"coef": 0.0, "every": 1}
        mixer = AttentionSpec(
            **sizes, scale=float(m["scale"]), window=_whole((m.get("mask") or {}).get("size", 0)),
            temp_coef=float(temp["coef"]), temp_every=_whole(temp["every"]), v_mix=bool(m.get("v_mix", False)),
        )
        if mixer.window < 0 or mixer.temp_every < 1:
            raise ValueError(f"layer {index}: window {mixer.window}, temperature every {mixer.temp_every}")
    else:
        raise ValueError(f"layer {index}: unknown mixer type {kind!r}")
    mlp, f = None, entry.get("mlp")
    if f is not None:
        if f.get("kind", "dense") != "dense":
            raise ValueError(f"layer {index}: unknown feed-forward kind {f.get('kind')!r}")
        mlp = DenseSpec(ff=_whole(f["ff"]))
        if mlp.ff < 1:
            raise ValueError(f"layer {index}: feed-forward of size {mlp.ff}")
    return LayerSpec(mixer, mlp)


@register_config("lefulorn", architecture="Lefulorn")
@dataclasses.dataclass
class LefulornConfig(ModelConfig):
    layers: List[Dict[str, Any]] = dataclasses.field(default_factory=list)
    block_prefix: str = "l"

    kernel_library: ClassVar[str] = "hybrid"
    unsupported: ClassVar[FrozenSet[str]] = frozenset({"adapters", "quantization", "tensor parallelism"})

    def __post_init__(self):
        super().__post_init__()
        self._specs = tuple(_parse_layer(i, e) for i, e in enumerate(self.layers))
        mixing = [i for i, s in enumerate(self._specs) if isinstance(s.mixer, AttentionSpec) and s.mixer.v_mix]
        self.first_mixing_layer = mixing[0] if mixing else None
        sizes = {(self._specs[i].mixer.kv_heads, self._specs[i].mixer.vdim) for i in mixing}
        if len({g * v for g, v in sizes}) > 1:
            raise ValueError(f"layers {mixing} mix values of different sizes")
        # the first mixing layer's values of a token travel beside its residual
        g, v = next(iter(sizes)) if len(mixing) > 1 else (0, 0)
        self.carried_values = g * v

    @classmethod
    def from_hf_dict(cls, d: Dict[str, Any], name_or_path: str = "") -> "LefulornConfig":
        layers = list(d["layers"])
        mixers = [e["mixer"] for e in layers]
        flat = {
            "hidden_size": int(d.get("width", d.get("hidden_size", 0))),
            "vocab_size": int(d.get("vocab", d.get("vocab_size", 0))),
            "layer_norm_eps": float(d["norm"]["eps"] if "norm" in d else d["layer_norm_eps"]),
            "num_hidden_layers": len(layers),
            "num_attention_heads": max((int(m["heads"]) for m in mixers), default=1),
            "num_key_value_heads": max((int(m.get("kv_heads", m["heads"])) for m in mixers), default=1),
            "intermediate_size": max((int(e["mlp"]["ff"]) for e in layers if e.get("mlp")), default=0),
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

    @property
    def stream_width(self) -> int:
        return self.hidden_size + self.carried_values

    @property
    def rewindable(self) -> bool:
        return not any(isinstance(s.mixer, DeltaSpec) for s in self._specs)

    def block_param_count(self) -> int:
        def count(s: LayerSpec) -> int:
            m, h = s.mixer, self.hidden_size
            wide = m.heads * m.vdim
            if isinstance(m, DeltaSpec):
                n = h * (2 * m.kv_heads * m.dim + 2 * wide + m.heads + m.dim + m.vdim)
                n += m.heads * (m.dim * m.dim + m.vdim * m.vdim)
            else:
                n = h * ((m.heads + m.kv_heads) * m.dim + m.kv_heads * m.vdim + 2 * wide)
            return n + (0 if s.mlp is None else 2 * h * s.mlp.ff)

        return max((count(s) for s in self._specs), default=1)

    def cache_values_per_token(self, block_index: int = 0) -> int:
        m = self._specs[block_index].mixer
        if isinstance(m, DeltaSpec):
            return 0
        return m.kv_heads * (-(-m.dim // KEY_PAD) * KEY_PAD + -(-m.vdim // VALUE_PAD) * VALUE_PAD)

    def state_shapes(self, block_index: int = 0) -> Dict[str, Tuple[int, ...]]:
        """delta: the recurrent matrix, padded for 16-wide tiles; conv: the last
        raw inputs of the short convolutions, position p in row p % taps."""
        m = self._specs[block_index].mixer
        if not isinstance(m, DeltaSpec):
            return {}
        return {
            "delta": (m.heads, -(-m.dim // 16) * 16, -(-m.vdim // 16) * 16),
            "conv": (m.taps, 2 * m.kv_heads * m.dim + m.heads * m.vdim),
        }
