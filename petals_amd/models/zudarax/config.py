"""Zudarax config: decoder layers whose attention and feed-forward read one norm,
described layer by layer.

config.json gives ``vocab``, ``width``, ``norm.eps``, ``norm.groups`` and a list
``layers``; each entry names its mixer (``type``), the mixer's own sizes and constants,
and its feed-forward (or null). The types differ in what happens to queries and keys,
how scores become weights and which keys are seen; a spec has a field for each of
these mechanisms, neutral where a type is without it. Nothing is uniform across layers.
"""

from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, FrozenSet, List, Optional, Tuple

import torch

from petals_amd.models.config_base import ModelConfig, register_config

KEY_PAD, VALUE_PAD = 32, 16  # head sizes in the cache are rounded up to these (ops/scores.py)


@dataclasses.dataclass(frozen=True)
class YarnSpec:
    """Frequencies divided by `factor` where a pair turns slowly over `original` positions."""

    factor: float
    original: float
    fast: float  # turns over `original` positions above which a frequency stays as it is
    slow: float  # and below which it is divided whole


@dataclasses.dataclass(frozen=True)
class RotarySpec:
    dims: int  # the first dimensions of a head that turn; the rest pass
    base: float
    yarn: Optional[YarnSpec] = None


@dataclasses.dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int  # query/key dimensions of one map of a head
    vdim: int
    scale: float
    rot: RotarySpec
    maps: int = 1  # weights per head: 2 are subtracted from one another
    taps: int = 0  # short convolution of queries, keys and values, the current token included; 0: none
    bias: bool = False  # of the projections
    qk_norm: bool = False  # over the whole projection, before rotation
    softcap: float = 0.0  # 0: scores are not capped
    chunk: int = 0  # position i sees those before it in its run of this many positions; 0: all
    sigmoid: bool = False  # weights are sigmoids of scores with a bias per head, not a softmax
    diff: float = 0.0  # constant of the second map's share
    head_gate: bool = False  # sigmoid of the layer's input, one number per head

    @property
    def dim_pad(self) -> int:
        return -(-self.dim // KEY_PAD) * KEY_PAD

    @property
    def vdim_pad(self) -> int:
        return -(-self.vdim // VALUE_PAD) * VALUE_PAD

    @property
    def columns(self) -> int:
        """Padded values of a token's queries, keys and values."""
        return self.maps * (self.heads + self.kv_heads) * self.dim_pad + self.kv_heads * self.vdim_pad


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    ff: int


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec
    mlp: Optional[DenseSpec]


def _whole(value) -> int:
    if int(value) != value:
        raise ValueError(f"{value!r} is not a whole number")
    return int(value)


def _rotary(index: int, rot: Dict[str, Any], dim: int) -> RotarySpec:
    dims, base, scaling = _whole(rot["dims"]), float(rot["base"]), rot.get("scaling")
    if dims % 2 or not 0 <= dims <= dim:
        raise ValueError(f"layer {index}: {dims} of {dim} dimensions cannot be rotated in pairs")
    yarn = None
    if scaling is not None:
        yarn = YarnSpec(**{name: float(scaling[name]) for name in ("factor", "original", "fast", "slow")})
        if min(dataclasses.astuple(yarn)) <= 0:
            raise ValueError(f"layer {index}: rotation scaling {scaling}")
    return RotarySpec(dims, base, yarn)


def _parse_layer(index: int, entry: Dict[str, Any]) -> LayerSpec:
    kind, m = entry.get("type"), entry["mixer"]
    sizes = {name: _whole(m[name]) for name in ("heads", "kv_heads", "dim", "vdim")}
    if min(sizes.values()) < 1 or sizes["heads"] % sizes["kv_heads"]:
        raise ValueError(f"layer {index}: mixer sizes {sizes}")
    common = dict(**sizes, scale=float(m["scale"]), rot=_rotary(index, m["rot"], sizes["dim"]))
    if kind == "attention":
        mixer = AttentionSpec(
            **common, taps=_whole(m["conv"]), bias=True, qk_norm=True, softcap=float(m["softcap"]),
            chunk=_whole(m["mask"]["size"]),
        )
        if mixer.chunk < 1 or mixer.softcap <= 0:
            raise ValueError(f"layer {index}: chunks of {mixer.chunk}, scores capped at {mixer.softcap}")
    elif kind == "attention_2":
        mixer = AttentionSpec(**common, maps=2, diff=float(m["diff"]), head_gate=True)
    elif kind == "attention_3":
        mixer = AttentionSpec(**common, taps=_whole(m["conv"]), sigmoid=True)
    else:
        raise ValueError(f"layer {index}: unknown mixer type {kind!r}")
    if "conv" in m and mixer.taps < 1:
        raise ValueError(f"layer {index}: a convolution of {mixer.taps} taps")
    mlp, f = None, entry.get("mlp")
    if f is not None:
        if f.get("kind", "dense") != "dense":
            raise ValueError(f"layer {index}: unknown feed-forward kind {f.get('kind')!r}")
        mlp = DenseSpec(ff=_whole(f["ff"]))
        if mlp.ff < 1:
            raise ValueError(f"layer {index}: feed-forward of size {mlp.ff}")
    return LayerSpec(mixer, mlp)


@register_config("zudarax", architecture="Zudarax")
@dataclasses.dataclass
class ZudaraxConfig(ModelConfig):
    layers: List[Dict[str, Any]] = dataclasses.field(default_factory=list)
    block_prefix: str = "l"
    norm_groups: int = 1  # equal parts of the residual, each normed by its own root mean square

    kernel_library: ClassVar[str] = "scores"
    unsupported: ClassVar[FrozenSet[str]] = frozenset({"adapters", "quantization", "tensor parallelism"})

    def __post_init__(self):
        super().__post_init__()
        self._specs = tuple(_parse_layer(i, e) for i, e in enumerate(self.layers))
        if self.norm_groups < 1 or self.hidden_size % self.norm_groups:
            raise ValueError(f"{self.hidden_size} values in {self.norm_groups} norm groups")

    @classmethod
    def from_hf_dict(cls, d: Dict[str, Any], name_or_path: str = "") -> "ZudaraxConfig":
        layers = list(d["layers"])
        mixers = [e["mixer"] for e in layers]
        norm = d.get("norm", {})
        flat = {
            "hidden_size": int(d.get("width", d.get("hidden_size", 0))),
            "vocab_size": int(d.get("vocab", d.get("vocab_size", 0))),
            "layer_norm_eps": float(norm["eps"] if "eps" in norm else d["layer_norm_eps"]),
            "norm_groups": _whole(norm.get("groups", d.get("norm_groups", 1))),
            "num_hidden_layers": len(layers),
            "num_attention_heads": max((int(m["heads"]) for m in mixers), default=1),
            "num_key_value_heads": max((int(m["kv_heads"]) for m in mixers), default=1),
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
    def rewindable(self) -> bool:
        """The convolutions' last inputs are not kept for every position."""
        return all(s.mixer.taps <= 1 for s in self._specs)

    def block_param_count(self) -> int:
        def count(s: LayerSpec) -> int:
            m, h = s.mixer, self.hidden_size
            n = h * (m.maps * (m.heads + m.kv_heads) * m.dim + (m.kv_heads + m.heads) * m.vdim)
            return n + (h * m.heads if m.head_gate else 0) + (0 if s.mlp is None else 2 * h * s.mlp.ff)

        return max((count(s) for s in self._specs), default=1)

    def cache_values_per_token(self, block_index: int = 0) -> int:
        """Padded keys, head by head and map by map, then padded values."""
        m = self._specs[block_index].mixer
        return m.kv_heads * (m.maps * m.dim_pad + m.vdim_pad)

    def state_shapes(self, block_index: int = 0) -> Dict[str, Tuple[int, ...]]:
        """conv: the last projected queries, keys and values, padded as in the
        projection; position p in row p % taps."""
        m = self._specs[block_index].mixer
        return {"conv": (m.taps, m.columns)} if m.taps > 1 else {}
