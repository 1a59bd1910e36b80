"""Native Zudarax decoder block, both sublayers side by side:

    h = norm1(x);   x <- x + (attention(h) + feed_forward(h))

with the residual x in 32-bit and a norm in equal parts. Attention is one of three
kinds: softmax over chunks with capped scores; the difference of two softmax maps;
sigmoid weights. Two of them run a short convolution over queries, keys and values,
whose last inputs are state of the sequence beside its cached keys and values.

Two forward contracts:
  * ``forward_paged(x, batch, pool)``: rows of any number of sequences, their keys,
    values and states in a PagedPool (server/paged_cache.py); x may be updated in
    place. The serving path: fused HIP kernels on the GPU (ops/scores.py), torch
    reference ops on the CPU.
  * ``forward(hidden)``: whole sequences [B, S, width], differentiable, no cache.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn.functional as F
from torch import nn

from petals_amd.models.zudarax.config import ZudaraxConfig
from petals_amd.ops import reference

_NAMES = {"norm1": "norm1", "up": "mlp.up", "down": "mlp.down", "act": "mlp.act"}


def _checkpoint_name(name: str) -> str:
    """q_bias -> mix.q.b, q_conv -> mix.q.conv, q_norm -> mix.q.norm, pb -> mix.pb"""
    base, _, kind = name.partition("_")
    return _NAMES.get(name) or f"mix.{base}" + {"": "", "bias": ".b", "conv": ".conv", "norm": ".norm"}[kind]


class ZudaraxBlock(nn.Module):
    paged = True
    _fast = None  # ops.scores.ScoresFastPath after optimize_for_inference()

    def __init__(self, config: ZudaraxConfig, layer_idx: int = 0):
        super().__init__()
        self.config = config
        self.layer_idx = self.source_layer = layer_idx
        spec = config.spec(layer_idx)
        self.mixer, self.mlp, self.eps, self.groups = spec.mixer, spec.mlp, config.layer_norm_eps, config.norm_groups
        m, d = spec.mixer, config.hidden_size

        def param(*shape):
            return nn.Parameter(torch.zeros(shape))

        self.norm1 = param(d)
        rows = {"q": m.heads * m.maps * m.dim, "k": m.kv_heads * m.maps * m.dim, "v": m.kv_heads * m.vdim}
        for name, n in rows.items():
            self.register_parameter(name, param(n, d))
            if m.bias:
                self.register_parameter(f"{name}_bias", param(n))
            if m.taps:
                self.register_parameter(f"{name}_conv", param(n, m.taps))
            if m.qk_norm and name != "v":
                self.register_parameter(f"{name}_norm", param(n))
        self.o = param(d, m.heads * m.vdim)
        if m.maps == 2:
            self.lq1, self.lk1, self.lq2, self.lk2 = (param(m.dim) for _ in range(4))
        if m.head_gate:
            self.g = param(m.heads, d)
        if m.sigmoid:
            self.pb = param(m.heads)
        if self.mlp is not None:
            self.up, self.down, self.act = param(self.mlp.ff, d), param(d, self.mlp.ff), param(4)

    # what server/from_pretrained.py leaves at 0 in random weights
    neutral_at_zero = frozenset({"lq1", "lk1", "lq2", "lk2", "pb"})

    def convert_state_dict(self, tensors: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors of this block (prefix removed) -> parameters. A
        missing or misshapen tensor is an error."""
        out = {}
        for name, p in self.named_parameters():
            theirs = _checkpoint_name(name)
            if theirs not in tensors:
                raise KeyError(f"block {self.layer_idx}: checkpoint has no tensor {theirs!r}")
            t = tensors[theirs]
            if tuple(t.shape) != tuple(p.shape):
                raise ValueError(f"block {self.layer_idx}: {theirs} is {tuple(t.shape)}, config says {tuple(p.shape)}")
            out[name] = t
        return out

    def optimize_for_inference(self, quant: str = "none") -> "ZudaraxBlock":
        """Repack the weights for the HIP kernels (frees the originals)."""
        from petals_amd.ops.scores import ScoresFastPath

        if quant != "none":
            raise ValueError(f"zudarax blocks are served in bfloat16 or float32, not quantized ({quant!r})")
        self._fast = ScoresFastPath(self)
        return self

    # ------------------------------------------------------------ cache spec

    def paged_cache_width(self) -> Optional[int]:
        return self.config.cache_values_per_token(self.layer_idx)

    def state_shapes(self):
        return self.config.state_shapes(self.layer_idx)

    def weight(self, name: str) -> torch.Tensor:
        return getattr(self, name) if self._fast is None else self._fast.weight(name)

    # --------------------------------------------------------------- serving

    def forward_paged(self, x: torch.Tensor, batch, pool) -> torch.Tensor:
        """x [T, D] 32-bit residual of the batch's rows; returns the new one."""
        state = pool.state(self.layer_idx)["conv"] if self.mixer.taps > 1 else None
        if self._fast is not None:
            return self._fast.forward_paged(x, batch, pool.layer(self.layer_idx), state)
        if x.is_cuda:
            raise RuntimeError("a block on the GPU needs optimize_for_inference() before it serves")
        m, cache = self.mixer, pool.layer(self.layer_idx)
        h = self._normed(x)
        raw = self._project(h)
        out = torch.empty(len(x), m.heads * m.vdim)
        wide = m.kv_heads * m.maps * m.dim_pad
        keys = cache[..., :wide].unflatten(-1, (m.kv_heads * m.maps, m.dim_pad))[..., : m.dim]
        values = cache[..., wide:].unflatten(-1, (m.kv_heads, m.vdim_pad))[..., : m.vdim]
        for s, (lo, hi) in enumerate(batch.row_ranges()):
            start, n = batch.starts[s], hi - lo
            before = None if state is None else self._swap_inputs(state[batch.slots[s]], start, raw, lo, hi)
            pos = torch.arange(start, start + n)
            q, k, v = self._qkv({name: t[None, lo:hi] for name, t in raw.items()}, before, pos)
            page, at = torch.as_tensor(batch.pages[s])[pos // cache.shape[1]], pos % cache.shape[1]
            keys[page, at], values[page, at] = k[0].flatten(1, 2).to(cache.dtype), v[0].to(cache.dtype)
            first = start // m.chunk * m.chunk if m.chunk else 0
            seen = torch.arange(first, start + n)
            page, at = torch.as_tensor(batch.pages[s])[seen // cache.shape[1]], seen % cache.shape[1]
            ks = keys[page, at].unflatten(1, (m.kv_heads, m.maps))
            out[lo:hi] = self._attend(q[0], ks, values[page, at], pos, seen)
        return self._rest(x, h, out)

    def _swap_inputs(self, ring, start, raw, lo, hi):
        """The convolution's inputs ahead of rows lo:hi, and theirs into the ring."""
        m = self.mixer
        heads = {"q": (m.heads * m.maps, m.dim, m.dim_pad), "k": (m.kv_heads * m.maps, m.dim, m.dim_pad),
                 "v": (m.kv_heads, m.vdim, m.vdim_pad)}
        views = dict(zip(heads, ring.split([n * padded for n, _, padded in heads.values()], dim=-1)))
        at = torch.arange(start - m.taps + 1, start)
        last = torch.arange(max(lo, hi - m.taps), hi)
        before = {}
        for name, (n, size, padded) in heads.items():
            rows = views[name].unflatten(-1, (n, padded))[..., :size]
            before[name] = torch.where((at >= 0)[:, None], rows[at % m.taps].flatten(1), torch.zeros(()))[None]
            rows[(last - lo + start) % m.taps] = raw[name][last].float().unflatten(-1, (n, size))
        return before

    # ----------------------------------------------------- stateless forward

    def forward(
        self,
        hidden_states: torch.Tensor,
        kv_cache=None,
        prefix_length: int = 0,
        ctx=None,
        shared=None,
    ) -> torch.Tensor:
        assert kv_cache is None and prefix_length == 0, "cached inference goes through forward_paged"
        x = hidden_states.float()
        h = self._normed(x)
        pos = torch.arange(x.shape[1], device=x.device)
        return self._rest(x, h, self._attend(*self._qkv(self._project(h), None, pos), pos, pos))

    # ----------------------------------------------------------------- parts

    def _normed(self, x: torch.Tensor) -> torch.Tensor:
        y = reference.group_rms_norm(x, self.weight("norm1").float(), self.groups, self.eps)
        return y.to(self.weight("o").dtype)

    def _project(self, h) -> Dict[str, torch.Tensor]:
        raw = {}
        for name in "qkv":
            raw[name] = (h @ self.weight(name).T).float()
            if self.mixer.bias:
                raw[name] = raw[name] + self.weight(f"{name}_bias").float()
        return raw

    def _qkv(self, raw, before, pos):
        """Projections [B, S, rows] at positions pos, the convolution's inputs ahead of them or
        None -> q [B, S, H, maps, dim], k [B, S, G, maps, dim], v [B, S, G, vdim]."""
        m, w, out = self.mixer, self.weight, {}
        freqs, factor = reference.rotary_frequencies(m.rot.dims, m.rot.base, m.rot.yarn, pos.device)
        for name, heads in (("q", m.heads), ("k", m.kv_heads), ("v", m.kv_heads)):
            x = raw[name]
            if m.taps:
                x = F.pad(x, (0, 0, m.taps - 1, 0)) if before is None else torch.cat([before[name], x], dim=1)
                x = reference.short_conv(x, w(f"{name}_conv").float())
            if name == "v":
                out[name] = x.unflatten(-1, (heads, m.vdim))
                continue
            if m.qk_norm:
                x = reference.rms_norm(x, w(f"{name}_norm").float(), self.eps)
            x = x.unflatten(-1, (heads, m.maps, m.dim))
            out[name] = reference.rotate_pairs(x, pos[:, None, None], freqs, factor)
        return out["q"], out["k"], out["v"]

    def _attend(self, q, k, v, q_pos, k_pos):
        """[..., Sq, H * vdim], 32-bit, not yet gated"""
        m = self.mixer
        seen = reference.visible(q_pos, k_pos, chunk=m.chunk)
        maps = [
            reference.scored_attention(
                q[..., n, :], k[..., n, :], v, seen, scale=m.scale, softcap=m.softcap,
                sigmoid_bias=self.weight("pb") if m.sigmoid else None,
            )
            for n in range(m.maps)
        ]
        if m.maps == 2:
            share = reference.differential_share(*(self.weight(n) for n in ("lq1", "lk1", "lq2", "lk2")), m.diff)
            maps[0] = reference.rms_norm(maps[0] - share * maps[1], maps[0].new_ones(()), self.eps) * (1.0 - m.diff)
        return maps[0].flatten(-2)

    def _rest(self, x, h, y):
        """x, its norm and the attended values -> the block's output."""
        m, w = self.mixer, self.weight
        if m.head_gate:
            y = (y.unflatten(-1, (m.heads, m.vdim)) * torch.sigmoid((h @ w("g").T).float())[..., None]).flatten(-2)
        add = (y.to(h.dtype) @ w("o").T).float()
        if self.mlp is not None:
            a = reference.poly_norm((h @ w("up").T).float(), w("act").float(), self.eps).to(h.dtype)
            add = add + (a @ w("down").T).float()
        return x + add
