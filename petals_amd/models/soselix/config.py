"""Soselix config: pre-norm decoder layers that mix tokens with latent attention
(rotated key part, sink, output gate), HGRN2 or Mamba-2, described layer by layer.

config.json gives ``vocab``, ``width``, ``norm.eps``, ``residual_mult``,
``embedding.scale`` and a list ``layers``; each entry names its mixer (``type``),
the mixer's own sizes and constants, and its feed-forward (or null). Nothing is
uniform across layers.
"""

from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, FrozenSet, List, Optional, Tuple, Union

import torch

from petals_amd.models.config_base import ModelConfig, register_config

LATENT_PAD, STATE_PAD = 32, 16  # sizes in the cache and in the state are rounded up to these (ops/recurrent.py)


@dataclasses.dataclass(frozen=True)
class LatentAttentionSpec:
    """Latent (MLA-style) attention with a rotated key part that all heads share."""

    heads: int
    dim: int  # query/key dimensions per head that come from the latent
    rot_dim: int  # query/key dimensions per head that are rotated
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_turned: int  # the first of the rot_dim dimensions that turn; the rest pass
    kv_from: Optional[int]  # layer whose cached rows are read (None: its own)

    @property
    def latent_pad(self) -> int:
        return -(-self.kv_rank // LATENT_PAD) * LATENT_PAD

    @property
    def rot_pad(self) -> int:
        return -(-self.rot_dim // LATENT_PAD) * LATENT_PAD


@dataclasses.dataclass(frozen=True)
class Hgrn2Spec:
    """Linear attention whose forget gate also decides what is written."""

    heads: int
    dim: int
    vdim: int


@dataclasses.dataclass(frozen=True)
class Mamba2Spec:
    """State-space duality: one decay per head, keys and queries per group of heads."""

    heads: int
    vdim: int
    state: int
    groups: int
    taps: int  # short convolution, the current token included
    norm_groups: int

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:  # of the convolution
        return self.inner + 2 * self.groups * self.state


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    ff: int


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: Union[LatentAttentionSpec, Hgrn2Spec, Mamba2Spec]
    mlp: Optional[DenseSpec]


def _whole(value) -> int:
    if int(value) != value:
        raise ValueError(f"{value!r} is not a whole number")
    return int(value)


def _sizes(index: int, source: Dict[str, Any], **names: str) -> Dict[str, int]:
    sizes = {ours: _whole(source[theirs]) for ours, theirs in names.items()}
    if min(sizes.values()) < 1:
        raise ValueError(f"layer {index}: sizes must be positive: {sizes}")
    return sizes


def _parse_layer(index: int, entry: Dict[str, Any]) -> LayerSpec:
    kind, m = entry.get("type"), entry["mixer"]
    if kind == "latent_attention":
        sizes = _sizes(
            index, m, heads="heads", dim="dim", rot_dim="rot_dim", vdim="vdim", q_rank="q_rank", kv_rank="kv_rank"
        )
        turned = _whole(m["rot"].get("dims", sizes["rot_dim"]))
        if turned % 2 or not 0 <= turned <= sizes["rot_dim"]:
            raise ValueError(f"layer {index}: {turned} of {sizes['rot_dim']} dimensions cannot be rotated in pairs")
        mixer = LatentAttentionSpec(
            **sizes, scale=float(m["scale"]), rot_base=float(m["rot"]["base"]), rot_turned=turned,
            kv_from=None if m.get("kv_from") is None else _whole(m["kv_from"]),
        )
    elif kind == "hgrn2":
        mixer = Hgrn2Spec(**_sizes(index, m, heads="heads", dim="dim", vdim="vdim"))
    elif kind == "mamba2":
        mixer = Mamba2Spec(**_sizes(
            index, {"groups": 1, "norm_groups": 1, **m}, heads="heads", vdim="vdim", state="state", groups="groups",
            taps="conv", norm_groups="norm_groups",
        ))
        if mixer.heads % mixer.groups or mixer.inner % mixer.norm_groups:
            raise ValueError(
                f"layer {index}: {mixer.heads} heads in {mixer.groups} groups, "
                f"{mixer.inner} values in {mixer.norm_groups} norm groups"
            )
    else:
        raise ValueError(f"layer {index}: unknown mixer type {kind!r}")
    mlp, f = None, entry.get("mlp")
    if f is not None:
        if f.get("kind", "dense") != "dense":
            raise ValueError(f"layer {index}: unknown feed-forward kind {f.get('kind')!r}")
        mlp = DenseSpec(**_sizes(index, f, ff="ff"))
    return LayerSpec(mixer, mlp)


@register_config("soselix", architecture="Soselix")
@dataclasses.dataclass
class SoselixConfig(ModelConfig):
    layers: List[Dict[str, Any]] = dataclasses.field(default_factory=list)
    block_prefix: str = "l"
    residual_mult: float = 1.0  # factor of what a sublayer adds to the residual
    embedding_scale: float = 1.0

    kernel_library: ClassVar[str] = "recurrent"
    unsupported: ClassVar[FrozenSet[str]] = frozenset({"adapters", "quantization", "tensor parallelism"})

    def __post_init__(self):
        super().__post_init__()
        self._specs = tuple(_parse_layer(i, e) for i, e in enumerate(self.layers))
        for i, spec in enumerate(self._specs):
            source = getattr(spec.mixer, "kv_from", None)
            if source is None:
                continue
            m = spec.mixer
            o = self._specs[source].mixer if 0 <= source < i else None
            if not isinstance(o, LatentAttentionSpec) or o.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from {source} must be an earlier layer with a latent of its own")
            if (o.kv_rank, o.rot_dim, o.rot_base, o.rot_turned) != (m.kv_rank, m.rot_dim, m.rot_base, m.rot_turned):
                raise ValueError(f"layer {i}: latent size or rotation differs from that of layer {source}")

    @classmethod
    def from_hf_dict(cls, d: Dict[str, Any], name_or_path: str = "") -> "SoselixConfig":
        layers = list(d["layers"])
        flat = {
            "hidden_size": int(d.get("width", d.get("hidden_size", 0))),
            "vocab_size": int(d.get("vocab", d.get("vocab_size", 0))),
            "layer_norm_eps": float(d["norm"]["eps"] if "norm" in d else d["layer_norm_eps"]),
            "embedding_scale": float(d["embedding"]["scale"] if "embedding" in d else d.get("embedding_scale", 1.0)),
            "num_hidden_layers": len(layers),
            "num_attention_heads": max((int(e["mixer"]["heads"]) for e in layers), default=1),
            "num_key_value_heads": 1,
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
        return all(isinstance(s.mixer, LatentAttentionSpec) for s in self._specs)

    def valid_cuts(self) -> Optional[FrozenSet[int]]:
        """A cut at c separates blocks < c from blocks >= c; none may fall
        between a layer and the layer whose cache it reads."""
        cuts = set(range(len(self._specs) + 1))
        for i, spec in enumerate(self._specs):
            source = getattr(spec.mixer, "kv_from", None)
            if source is not None:
                cuts -= set(range(source + 1, i + 1))
        return frozenset(cuts)

    def block_param_count(self) -> int:
        def count(s: LayerSpec) -> int:
            m, h = s.mixer, self.hidden_size
            n = h * m.heads * m.vdim
            if isinstance(m, LatentAttentionSpec):
                n += m.q_rank * (h + m.heads * (m.dim + m.rot_dim)) + m.heads * (h + m.kv_rank * (m.dim + m.vdim))
                if m.kv_from is None:
                    n += h * (m.kv_rank + m.rot_dim)
            elif isinstance(m, Hgrn2Spec):
                n += h * m.heads * (2 * m.dim + m.vdim)
            else:
                n += h * (m.inner + m.channels + m.heads)
            return n + (0 if s.mlp is None else 2 * h * s.mlp.ff)

        return max((count(s) for s in self._specs), default=1)

    def cache_values_per_token(self, block_index: int = 0) -> int:
        """A latent row, then the rotated key part, both padded."""
        m = self._specs[block_index].mixer
        if not isinstance(m, LatentAttentionSpec) or m.kv_from is not None:
            return 0
        return m.latent_pad + m.rot_pad

    def state_shapes(self, block_index: int = 0) -> Dict[str, Tuple[int, ...]]:
        """matrix: the recurrent state, padded for 16-wide tiles; conv: the last
        raw inputs of the short convolution, position p in row p % taps."""
        m = self._specs[block_index].mixer
        if isinstance(m, LatentAttentionSpec):
            return {}
        rows = m.dim if isinstance(m, Hgrn2Spec) else m.state
        shapes = {"matrix": (m.heads, -(-rows // STATE_PAD) * STATE_PAD, -(-m.vdim // STATE_PAD) * STATE_PAD)}
        if isinstance(m, Mamba2Spec):
            shapes["conv"] = (m.taps, m.channels)
        return shapes
