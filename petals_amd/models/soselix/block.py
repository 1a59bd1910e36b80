"""Native Soselix decoder block, pre-norm:

    x <- x + m mixer(norm1(x));   x <- x + m feed_forward(norm2(x))

with the residual x in 32-bit and norms that have one weight for all coordinates.
The mixer is latent attention over cached latents and rotated key parts, HGRN2, or
Mamba-2; the last two keep one matrix per head and sequence, Mamba-2 also a few
rows of convolution inputs.

A block with ``kv_from`` owns no cache and reads the rows of an earlier block,
which must be served by the same server in the same session
(SoselixConfig.valid_cuts).

Two forward contracts:
  * ``forward_paged(x, batch, pool)``: rows of any number of sequences, their
    latents and states in a PagedPool (server/paged_cache.py); x may be updated in
    place. The serving path: fused HIP kernels on the GPU (ops/recurrent.py), torch
    reference ops on the CPU.
  * ``forward(hidden, shared=...)``: whole sequences [B, S, D], differentiable,
    no cache; ``shared`` carries cached rows between the blocks of one chain.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn.functional as F
from torch import nn

from petals_amd.models.soselix.config import Hgrn2Spec, LatentAttentionSpec, SoselixConfig
from petals_amd.ops import reference

# parameter -> checkpoint tensor, behind the block's prefix
_NAMES = {
    "latent": {
        "dq": "mix.dq", "dq_norm": "mix.dq.norm", "uq": "mix.uq", "dkv": "mix.dkv", "dkv_norm": "mix.dkv.norm",
        "uk": "mix.uk", "uv": "mix.uv", "sink": "mix.sink", "g": "mix.g",
    },
    "hgrn": {
        "q": "mix.q", "f": "mix.f", "f_bias": "mix.f.b", "lower": "mix.lower", "v": "mix.v", "head_norm": "mix.norm",
    },
    "mamba": {
        "in_proj": "mix.in", "conv": "mix.conv", "conv_bias": "mix.conv.b", "dt_bias": "mix.dt_bias",
        "A_log": "mix.A_log", "D": "mix.D", "group_norm": "mix.norm",
    },
    "every": {
        "norm1": "norm1", "norm2": "norm2", "o": "mix.o", "up": "mlp.up", "up_bias": "mlp.up.b", "down": "mlp.down",
        "down_bias": "mlp.down.b", "act": "mlp.act",
    },
}


class SoselixBlock(nn.Module):
    paged = True
    _fast = None  # ops.recurrent.RecurrentFastPath after optimize_for_inference()

    def __init__(self, config: SoselixConfig, layer_idx: int = 0):
        super().__init__()
        self.config = config
        self.layer_idx = self.source_layer = layer_idx
        spec = config.spec(layer_idx)
        self.mixer, self.mlp, self.eps, self.mult = spec.mixer, spec.mlp, config.layer_norm_eps, config.residual_mult
        m, d = spec.mixer, config.hidden_size

        def param(*shape):
            return nn.Parameter(torch.zeros(shape))

        self.norm1 = param()
        self.o = param(d, m.heads * m.vdim)
        if isinstance(m, LatentAttentionSpec):
            self.kind = "latent"
            self.dq, self.dq_norm = param(m.q_rank, d), param(m.q_rank)
            self.uq = param(m.heads * (m.dim + m.rot_dim), m.q_rank)
            if m.kv_from is None:
                self.dkv, self.dkv_norm = param(m.kv_rank + m.rot_dim, d), param(m.kv_rank)
            else:
                self.source_layer = m.kv_from
            self.uk, self.uv = param(m.heads * m.dim, m.kv_rank), param(m.heads * m.vdim, m.kv_rank)
            self.sink, self.g = param(m.heads), param(m.heads, d)
        elif isinstance(m, Hgrn2Spec):
            self.kind = "hgrn"
            n = m.heads * m.dim
            self.q, self.f, self.v = param(n, d), param(n, d), param(m.heads * m.vdim, d)
            self.f_bias, self.lower, self.head_norm = param(n), param(n), param(m.vdim)
        else:
            self.kind = "mamba"
            self.in_proj = param(m.inner + m.channels + m.heads, d)
            self.conv, self.conv_bias = param(m.channels, m.taps), param(m.channels)
            self.dt_bias, self.A_log, self.D = param(m.heads), param(m.heads), param(m.heads)
            self.group_norm = param(m.inner)
        if self.mlp is not None:
            self.norm2 = param()
            self.up, self.up_bias = param(self.mlp.ff, d), param(self.mlp.ff)
            self.down, self.down_bias = param(d, self.mlp.ff), param(d)
            self.act = param(2)

    # what server/from_pretrained.py leaves at 0 in random weights
    neutral_at_zero = frozenset({"sink", "lower", "A_log", "act"})

    def convert_state_dict(self, tensors: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint tensors of this block (prefix removed) -> parameters. A
        missing or misshapen tensor is an error."""
        names, out = {**_NAMES["every"], **_NAMES[self.kind]}, {}
        for name, p in self.named_parameters():
            if names[name] not in tensors:
                raise KeyError(f"block {self.layer_idx}: checkpoint has no tensor {names[name]!r}")
            t = tensors[names[name]]
            if p.dim() == 0 and t.numel() == 1:
                t = t.reshape(())
            if tuple(t.shape) != tuple(p.shape):
                raise ValueError(
                    f"block {self.layer_idx}: {names[name]} is {tuple(t.shape)}, config says {tuple(p.shape)}"
                )
            out[name] = t
        return out

    def optimize_for_inference(self, quant: str = "none") -> "SoselixBlock":
        """Repack the weights for the HIP kernels (frees the originals)."""
        from petals_amd.ops.recurrent import RecurrentFastPath

        if quant != "none":
            raise ValueError(f"soselix blocks are served in bfloat16 or float32, not quantized ({quant!r})")
        self._fast = RecurrentFastPath(self)
        return self

    # ------------------------------------------------------------ cache spec

    def paged_cache_width(self) -> Optional[int]:
        """Padded size of the rows this block OWNS in the pages; None if it has none."""
        return self.config.cache_values_per_token(self.layer_idx) or None

    def state_shapes(self):
        return self.config.state_shapes(self.layer_idx)

    def weight(self, name: str) -> torch.Tensor:
        return getattr(self, name) if self._fast is None else self._fast.weight(name)

    # --------------------------------------------------------------- serving

    def forward_paged(self, x: torch.Tensor, batch, pool) -> torch.Tensor:
        """x [T, D] 32-bit residual of the batch's rows; returns the new one."""
        if self._fast is not None:
            if self.kind == "latent":
                return self._fast.forward_paged(x, batch, cache=pool.layer(self.source_layer))
            return self._fast.forward_paged(x, batch, state=pool.state(self.layer_idx))
        if x.is_cuda:
            raise RuntimeError("a block on the GPU needs optimize_for_inference() before it serves")
        h = self._normed(x, self.norm1)
        if self.kind == "latent":
            y = self._latent_paged(h, batch, pool.layer(self.source_layer))
        else:
            y = self._recurrent_paged(h, batch, pool.state(self.layer_idx))
        return self._rest(x, h, y)

    def _latent_paged(self, h, batch, cache):
        m = self.mixer
        pos = torch.cat([torch.arange(s, s + n) for s, n in zip(batch.starts, batch.lens)])
        if m.kv_from is None:
            c, turned = self._latent_rows(h, pos)
            reference.paged_write(cache, batch, c)
            reference.paged_write(cache[..., m.latent_pad :], batch, turned)
        q = self._queries(h, pos)
        out = torch.empty(len(h), m.heads * m.vdim)
        for s, (lo, hi) in enumerate(batch.row_ranges()):
            seen = torch.arange(batch.starts[s] + hi - lo)
            rows = cache[torch.as_tensor(batch.pages[s])[seen // cache.shape[1]], seen % cache.shape[1]].to(h.dtype)
            c, turned = rows[:, : m.kv_rank], rows[:, m.latent_pad : m.latent_pad + m.rot_dim]
            out[lo:hi] = self._attend(q[lo:hi], c, turned, pos[lo:hi], seen)
        return out

    def _recurrent_paged(self, h, batch, state):
        m = self.mixer
        out = torch.empty(len(h), m.heads * m.vdim)
        for slot, start, (lo, hi) in zip(batch.slots, batch.starts, batch.row_ranges()):
            rows = m.dim if self.kind == "hgrn" else m.state
            matrix = state["matrix"][slot][:, :rows, : m.vdim]
            before = matrix.clone()[None] if start else None
            if self.kind == "hgrn":
                y, last = self._hgrn(h[None, lo:hi], before)
            else:
                ring = state["conv"][slot]
                at = torch.arange(start - m.taps + 1, start)
                inputs = torch.where((at >= 0)[:, None], ring[at % m.taps], torch.zeros(()))
                y, last, inputs = self._mamba(h[None, lo:hi], before, inputs[None])
                n = min(hi - lo, m.taps)
                ring[torch.arange(start + hi - lo - n, start + hi - lo) % m.taps] = inputs[0, inputs.shape[1] - n :]
            matrix.copy_(last[0])
            out[lo:hi] = y[0]
        return out

    # ----------------------------------------------------- stateless forward

    def forward(
        self,
        hidden_states: torch.Tensor,
        kv_cache=None,
        prefix_length: int = 0,
        ctx=None,
        shared: Optional[Dict[int, tuple]] = None,
    ) -> torch.Tensor:
        assert kv_cache is None and prefix_length == 0, "cached inference goes through forward_paged"
        m = self.mixer
        b, s, _ = hidden_states.shape
        x = hidden_states.float()
        h = self._normed(x, self.weight("norm1"))
        if self.kind == "latent":
            pos = torch.arange(s, device=x.device)
            if m.kv_from is None:
                rows = tuple(t.to(h.dtype) for t in self._latent_rows(h, pos))
                if shared is not None:
                    shared[self.layer_idx] = rows
            elif shared is None or m.kv_from not in shared:
                raise ValueError(f"block {self.layer_idx} needs the latent of block {m.kv_from} from the same chain")
            else:
                rows = shared[m.kv_from]
            y = self._attend(self._queries(h, pos), *rows, pos, pos)
        elif self.kind == "hgrn":
            y, _ = self._hgrn(h, None)
        else:
            y, _, _ = self._mamba(h, None, torch.zeros(b, m.taps - 1, m.channels, device=x.device))
        return self._rest(x, h, y)

    # ----------------------------------------------------------------- parts

    def _normed(self, x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
        return reference.rms_norm(x, weight.float(), self.eps).to(self.weight("o").dtype)

    def _latent_rows(self, h, pos):
        """(latent, rotated key part) of each row, 32-bit."""
        m = self.mixer
        y = (h @ self.weight("dkv").T).float()
        c = reference.rms_norm(y[..., : m.kv_rank], self.weight("dkv_norm").float(), self.eps)
        return c, reference.rotate_halves(y[..., m.kv_rank :], pos, m.rot_turned, m.rot_base)

    def _queries(self, h, pos):
        m = self.mixer
        cq = reference.rms_norm((h @ self.weight("dq").T).float(), self.weight("dq_norm").float(), self.eps).to(h.dtype)
        q = (cq @ self.weight("uq").T).float().unflatten(-1, (m.heads, m.dim + m.rot_dim))
        turned = reference.rotate_halves(q[..., m.dim :], pos[:, None], m.rot_turned, m.rot_base)
        return torch.cat([q[..., : m.dim], turned], dim=-1)

    def _attend(self, q, c, turned, q_pos, k_pos):
        """q [..., Sq, H, dim + rot_dim] against cached rows [..., Sk, ...]: [..., Sq, H * vdim], not yet gated."""
        m = self.mixer
        k = (c @ self.weight("uk").T).float().unflatten(-1, (m.heads, m.dim))
        k = torch.cat([k, turned.float().unsqueeze(-2).expand(*k.shape[:-1], m.rot_dim)], dim=-1)
        v = (c @ self.weight("uv").T).unflatten(-1, (m.heads, m.vdim))
        return reference.biased_sink_attention(
            q, k, v, q_pos, k_pos, scale=m.scale, window=0, sink=self.weight("sink")
        ).flatten(-2)

    def _hgrn(self, h, state):
        """h [B, S, width] -> (o normed per head, last state)."""
        m, w = self.mixer, self.weight
        q = F.silu((h @ w("q").T).float()).unflatten(-1, (m.heads, m.dim))
        v = (h @ w("v").T).float().unflatten(-1, (m.heads, m.vdim))
        k, f = reference.forget_gate((h @ w("f").T).float() + w("f_bias").float(), w("lower").float())
        k, f = (t.unflatten(-1, (m.heads, m.dim)) for t in (k, f))
        o, last = reference.gated_linear_attention(q, k, v, f, state)
        return reference.rms_norm(o, w("head_norm").float(), self.eps).flatten(-2), last

    def _mamba(self, h, state, before):
        """h [B, S, width] -> (y gated and normed, last state, convolution inputs with `before`)."""
        m, w = self.mixer, self.weight
        z, raw, dt = (h @ w("in_proj").T).float().split([m.inner, m.channels, m.heads], dim=-1)
        raw = torch.cat([before, raw], dim=1)
        mixed = F.silu(reference.short_conv(raw, w("conv").float()) + w("conv_bias").float())
        x, b, c = mixed.split([m.inner, m.groups * m.state, m.groups * m.state], dim=-1)
        x = x.unflatten(-1, (m.heads, m.vdim))
        b, c = (
            t.unflatten(-1, (m.groups, m.state)).repeat_interleave(m.heads // m.groups, dim=-2) for t in (b, c)
        )
        dt = F.softplus(dt + w("dt_bias").float())
        decay = torch.exp(-torch.exp(w("A_log").float()) * dt)
        y, last = reference.gated_linear_attention(c, b, dt[..., None] * x, decay[..., None], state)
        y = (y + w("D").float()[:, None] * x).flatten(-2) * F.silu(z)
        return reference.group_rms_norm(y, w("group_norm").float(), m.norm_groups, self.eps), last, raw

    def _rest(self, x, h, y):
        """x and the mixer's output before its last projection (attention: before its gate) -> the block's output."""
        w = self.weight
        if self.kind == "latent":
            y = y.unflatten(-1, (self.mixer.heads, -1)) * torch.sigmoid((h @ w("g").T).float())[..., None]
            y = y.flatten(-2)
        x = x + self.mult * (y.to(h.dtype) @ w("o").T).float()
        if self.mlp is None:
            return x
        h = self._normed(x, w("norm2"))
        p, q = w("act").float()
        a = reference.xielu((h @ w("up").T).float() + w("up_bias").float(), p, q).to(h.dtype)
        return x + self.mult * ((a @ w("down").T).float() + w("down_bias").float())
