"""Native Lefulorn decoder block, pre-norm:

    x <- x + mixer(norm1(x));   x <- x + feed_forward(norm2(x))

with the residual x in 32-bit. The mixer is a gated delta rule with a decay per
key channel, whose state is one matrix per head and a few rows of convolution
inputs per sequence, or windowed attention over cached keys and values.

The stream between blocks holds the residual and, beside it, the values of the
first layer that mixes values (config.stream_width), so that a chain may be cut
between any two blocks.

Two forward contracts:
  * ``forward_paged(x, batch, pool)``: rows of any number of sequences, their
    keys, values and states in a PagedPool (server/paged_cache.py); x may be
    updated in place. The serving path: fused HIP kernels on the GPU
    (ops/hybrid.py), torch reference ops on the CPU.
  * ``forward(hidden)``: whole sequences [B, S, stream width], differentiable,
    no cache.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn.functional as F
from torch import nn

from petals_amd.models.lefulorn.config import KEY_PAD, DeltaSpec, LefulornConfig
from petals_amd.ops import reference


class LefulornBlock(nn.Module):
    paged = True
    _fast = None  # ops.hybrid.HybridFastPath after optimize_for_inference()

    def __init__(self, config: LefulornConfig, layer_idx: int = 0):
        super().__init__()
        self.config = config
        self.layer_idx = self.source_layer = layer_idx
        spec = config.spec(layer_idx)
        self.mixer, self.mlp, self.eps = spec.mixer, spec.mlp, config.layer_norm_eps
        self.delta = isinstance(spec.mixer, DeltaSpec)
        m, d = spec.mixer, config.hidden_size
        # 'first': sets the values that later layers mix in; 'mix': mixes them in
        self.mix = None
        if not self.delta and m.v_mix and config.carried_values:
            self.mix = "first" if layer_idx == config.first_mixing_layer else "mix"

        def param(*shape):
            return nn.Parameter(torch.zeros(shape))

        self.norm1 = param(d)
        self.q = param((m.kv_heads if self.delta else m.heads) * m.dim, d)
        self.k = param(m.kv_heads * m.dim, d)
        self.v = param((m.heads if self.delta else m.kv_heads) * m.vdim, d)
        self.o = param(d, m.heads * m.vdim)
        if self.delta:
            for name in ("q", "k", "v"):
                self.register_parameter(f"{name}_conv", param(getattr(self, name).shape[0], m.taps))
            self.b = param(m.heads, d)
            self.A_log, self.dt_bias = param(m.heads), param(m.heads * m.dim)
            # the checkpoint gives the ranks (convert_state_dict)
            self.a1, self.a2 = param(m.dim, d), param(m.heads * m.dim, m.dim)
            self.g1, self.g2 = param(m.vdim, d), param(m.heads * m.vdim, m.vdim)
            self.o_norm = param(m.vdim)
        else:
            for name in ("q", "k", "v"):
                self.register_parameter(f"{name}_bias", param(getattr(self, name).shape[0]))
            self.sink = param(m.heads)
            self.g = param(m.heads * m.vdim, d)
            if m.v_mix:
                self.vmix = param()
        if self.mlp is not None:
            self.norm2 = param(d)
            self.up, self.up_bias = param(self.mlp.ff, d), param(self.mlp.ff)
            self.down, self.down_bias = param(d, self.mlp.ff), param(d)

    # what server/from_pretrained.py leaves at 0 in random weights
    neutral_at_zero = frozenset({"A_log", "sink", "vmix"})

    def convert_state_dict(self, tensors: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors of this block (prefix removed) -> parameters. A
        missing or misshapen tensor is an error."""
        special = {"o_norm": "mix.norm", "norm1": "norm1", "norm2": "norm2"}
        out = {}
        for name, p in list(self.named_parameters()):
            theirs = special.get(name)
            if theirs is None:
                base, _, kind = name.rpartition("_")
                part = "mlp" if name.split("_")[0] in ("up", "down") else "mix"
                theirs = f"{part}.{name}"
                if kind == "conv":
                    theirs = f"{part}.{base}.conv"
                elif kind == "bias" and base != "dt":
                    theirs = f"{part}.{base}.b"
            if theirs not in tensors:
                if name == "vmix" and self.mix != "mix":  # not used
                    out[name] = torch.zeros(())
                    continue
                raise KeyError(f"block {self.layer_idx}: checkpoint has no tensor {theirs!r}")
            out[name] = tensors[theirs].reshape(()) if name == "vmix" else tensors[theirs]
        if self.delta:
            for inner, outer in (("a1", "a2"), ("g1", "g2")):
                rank = out[inner].shape[0]
                shapes = {inner: (rank, self.config.hidden_size), outer: (getattr(self, outer).shape[0], rank)}
                for name, shape in shapes.items():
                    setattr(self, name, nn.Parameter(torch.empty(*shape, device="meta")))
        for name, p in self.named_parameters():
            if tuple(out[name].shape) != tuple(p.shape):
                raise ValueError(
                    f"block {self.layer_idx}: {name} is {tuple(out[name].shape)}, config says {tuple(p.shape)}"
                )
        return out

    def optimize_for_inference(self, quant: str = "none") -> "LefulornBlock":
        """Repack the weights for the HIP kernels (frees the originals)."""
        from petals_amd.ops.hybrid import HybridFastPath

        if quant != "none":
            raise ValueError(f"lefulorn blocks are served in bfloat16 or float32, not quantized ({quant!r})")
        self._fast = HybridFastPath(self)
        return self

    # ------------------------------------------------------------ cache spec

    def paged_cache_width(self) -> Optional[int]:
        """Values of one token in the pages: padded keys, then padded values; None for a recurrent layer."""
        return self.config.cache_values_per_token(self.layer_idx) or None

    def state_shapes(self):
        return self.config.state_shapes(self.layer_idx)

    def weight(self, name: str) -> torch.Tensor:
        return getattr(self, name) if self._fast is None else self._fast.weight(name)

    # --------------------------------------------------------------- serving

    def forward_paged(self, x: torch.Tensor, batch, pool) -> torch.Tensor:
        """x [T, stream width] 32-bit rows of the batch; returns the new ones."""
        if self._fast is not None:
            if self.delta:
                return self._fast.forward_paged(x, batch, state=pool.state(self.layer_idx))
            return self._fast.forward_paged(x, batch, cache=pool.layer(self.layer_idx))
        if x.is_cuda:
            raise RuntimeError("a block on the GPU needs optimize_for_inference() before it serves")
        d, m = self.config.hidden_size, self.mixer
        x, carried = x[:, :d], x[:, d:]
        h = self._normed(x, self.norm1)
        out = torch.empty(len(x), m.heads * m.vdim)
        if self.delta:
            state = pool.state(self.layer_idx)
            for slot, start, (lo, hi) in zip(batch.slots, batch.starts, batch.row_ranges()):
                matrix, conv = state["delta"][slot], state["conv"][slot]
                at = torch.arange(start - m.taps + 1, start) % m.taps
                before = conv[at] if start else torch.zeros_like(conv[at])
                if start < m.taps - 1:  # rows of positions before the first token
                    before = before * (torch.arange(start - m.taps + 1, start) >= 0)[:, None]
                own = matrix[:, : m.dim, : m.vdim] if start else None
                out[lo:hi], last, tail = self._delta_rule(h[None, lo:hi], own, before[None])
                matrix[:, : m.dim, : m.vdim] = last
                n = min(hi - lo, m.taps)
                conv[torch.arange(start + hi - lo - n, start + hi - lo) % m.taps] = tail[0, tail.shape[1] - n :]
        else:
            q, k, v = self._qkv(h)
            cache = pool.layer(self.layer_idx)
            if self.mix == "first":
                carried = v.float()
            elif self.mix == "mix":
                v = self._mixed(v, carried)
            wide = m.kv_heads * -(-m.dim // KEY_PAD) * KEY_PAD
            keys, values = cache[..., :wide], cache[..., wide:]
            reference.paged_write(keys.unflatten(-1, (m.kv_heads, -1))[..., : m.dim], batch, k.view(-1, m.kv_heads, m.dim))
            reference.paged_write(
                values.unflatten(-1, (m.kv_heads, -1))[..., : m.vdim], batch, v.view(-1, m.kv_heads, m.vdim)
            )
            for s, (lo, hi) in enumerate(batch.row_ranges()):
                start = batch.starts[s]
                first = max(0, start - m.window + 1) if m.window > 0 else 0
                pos = torch.arange(first, start + hi - lo)
                at = (torch.as_tensor(batch.pages[s])[pos // cache.shape[1]], pos % cache.shape[1])
                ks = keys[at].unflatten(-1, (m.kv_heads, -1))[..., : m.dim]
                vs = values[at].unflatten(-1, (m.kv_heads, -1))[..., : m.vdim]
                out[lo:hi] = self._attend(q[lo:hi], ks, vs, pos[start - first :], pos)
            out = out * torch.sigmoid((h @ self.g.T).float())
        x = self._feed_forward(x + (out.to(h.dtype) @ self.o.T).float())
        return torch.cat([x, carried], dim=1) if self.config.carried_values else x

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
        d, m = self.config.hidden_size, self.mixer
        b, s, _ = hidden_states.shape
        x, carried = hidden_states[..., :d].float(), hidden_states[..., d:].float()
        h = self._normed(x, self.weight("norm1"))
        if self.delta:
            channels = sum(self.weight(n).shape[0] for n in ("q", "k", "v"))
            before = torch.zeros(b, m.taps - 1, channels, device=x.device)
            y, _, _ = self._delta_rule(h, None, before)
        else:
            q, k, v = self._qkv(h)
            if self.mix == "first":
                carried = v.float()
            elif self.mix == "mix":
                v = self._mixed(v, carried)
            pos = torch.arange(s, device=x.device)
            y = self._attend(q, k.view(b, s, m.kv_heads, m.dim), v.view(b, s, m.kv_heads, m.vdim), pos, pos)
            y = y * torch.sigmoid((h @ self.weight("g").T).float())
        x = self._feed_forward(x + (y.to(h.dtype) @ self.weight("o").T).float())
        return torch.cat([x, carried], dim=-1)

    # ----------------------------------------------------------------- parts

    def _normed(self, x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
        return reference.rms_norm(x, weight.float(), self.eps).to(self.weight("o").dtype)

    def _delta_rule(self, h, state, before):
        """h [(B,) S, width] -> (o normed and gated, last state, convolution inputs with `before`)."""
        m, w = self.mixer, self.weight
        raw = torch.cat([h @ w(n).T for n in ("q", "k", "v")], dim=-1).float()
        raw = torch.cat([before, raw], dim=1)
        conv = F.silu(reference.short_conv(raw, torch.cat([w(f"{n}_conv") for n in ("q", "k", "v")]).float()))
        b, s = h.shape[:2]
        q, k, v = conv.split([m.kv_heads * m.dim, m.kv_heads * m.dim, m.heads * m.vdim], dim=-1)
        group = m.heads // m.kv_heads
        q, k = (
            reference.unit_vectors(t.view(b, s, m.kv_heads, m.dim)).repeat_interleave(group, dim=2) for t in (q, k)
        )
        beta = torch.sigmoid((h @ w("b").T).float())
        a = ((h @ w("a1").T) @ w("a2").T).float() + w("dt_bias").float()
        log_decay = -torch.exp(w("A_log").float())[:, None] * F.softplus(a).view(b, s, m.heads, m.dim)
        o, last = reference.gated_delta_rule(
            q * m.dim**-0.5, k, v.view(b, s, m.heads, m.vdim), log_decay.exp(), beta, state
        )
        gate = torch.sigmoid(((h @ w("g1").T) @ w("g2").T).float()).view(b, s, m.heads, m.vdim)
        o = reference.rms_norm(o, w("o_norm").float(), self.eps) * gate
        return o.reshape(b, s, -1), last, raw

    def _qkv(self, h):
        m = self.mixer
        q, k, v = ((h @ self.weight(n).T) + self.weight(f"{n}_bias").to(h.dtype) for n in ("q", "k", "v"))
        return q.unflatten(-1, (m.heads, m.dim)), k, v

    def _mixed(self, v, first):
        lam = self.weight("vmix").float()
        return ((1.0 - lam) * v.float() + lam * first).to(v.dtype)

    def _attend(self, q, k, v, q_pos, k_pos):
        m = self.mixer
        return reference.biased_sink_attention(
            q, k, v, q_pos, k_pos, scale=m.scale, window=m.window, sink=self.weight("sink"),
            slopes=reference.distance_slopes(m.heads, q.device),
            temperature=reference.query_temperature(q_pos, m.temp_coef, m.temp_every),
        ).flatten(-2)

    def _feed_forward(self, x):
        if self.mlp is None:
            return x
        w = self.weight
        h = self._normed(x, w("norm2"))
        a = F.linear(h, w("up"), w("up_bias").to(h.dtype)).relu().square()
        return x + F.linear(a, w("down"), w("down_bias").to(h.dtype)).float()
