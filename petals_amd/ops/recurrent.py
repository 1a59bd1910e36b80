"""MI355X fast path of pre-norm blocks with gated linear attention (HGRN2, Mamba-2)
or with latent attention whose keys have a rotated part (models/soselix).

Kernels: ops/csrc/linear_attn.hip, latent_attn.hip, rotary_latent.hip, prenorm.hip,
gemv.hip, in a library of their own (ops/build.py "recurrent").

Everything that reads the normed input is one product: queries, forget gate and
values; gate, convolution inputs and step sizes; query latent, key/value latent and
output gate. Latent attention works in latent space: W_uk is applied to the query and
W_uv to the attended latent, so attention reads the cached rows themselves, all heads
share them, and prompts and decoding take the same steps. A cached row is the latent
and, behind it, the rotated key part; only the latent is summed. Recurrent layers have
a kernel for batches of single tokens and chunked ones for all others. Packing and
routes: ops/packed.py.
"""

from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from petals_amd.ops.packed import _EPI_RAW, CHUNK, PackedBlock
from petals_amd.ops.packed import round_up as _up


def hip():
    """The compiled kernels; on a GPU there is nothing else to fall back to."""
    from petals_amd.ops import _hip

    return _hip.first_loaded("recurrent")


class RecurrentFastPath(PackedBlock):
    def __init__(self, block):
        super().__init__(block, hip())
        self.kind, self.mult = block.kind, block.mult
        self.norm1 = self._single(block, "norm1")
        self.run, pack = {
            "latent": (self._latent, self._pack_latent),
            "hgrn": (self._forget, self._pack_forget),
            "mamba": (self._ssm, self._pack_ssm),
        }[block.kind]
        pack(block)
        if self.mlp is not None:
            self.norm2 = self._single(block, "norm2")
            p, q = self._f32(block, "act").double()
            # z > 0: first z^2 + z/2;  z <= 0: second (exp(z) - 1 - z) + z/2
            self.xielu = (F.softplus(p).item(), 0.5 + F.softplus(q).item())
        self._finish(block)

    # ---------------------------------------------------------------- weights

    def _single(self, block, name):
        """A norm's one weight, as the vector that the kernels take."""
        return self._f32(block, name).expand(self.d).contiguous()

    def weight(self, name: str) -> torch.Tensor:
        if name == "in_proj":
            return torch.cat([self._views[n] for n in ("in_z", "in_conv", "in_dt")])
        if name == "uq":
            plain, turned = self._views["uq_plain"], self._views["uq_turned"]
            return torch.cat([plain, turned], dim=1).flatten(0, 1)
        return super().weight(name)

    def _pack_latent(self, block):
        m, d = self.spec, self.d
        parts = [("dq", 1, m.q_rank, m.q_rank), ("g", m.heads, 1, 1)]
        if m.kv_from is None:
            parts.append(("dkv", 1, m.kv_rank + m.rot_dim, m.kv_rank + m.rot_dim))
        self.at_q, self.at_g, *self.at_kv = self._columns(block, parts)
        self.q_norm = self._f32(block, "dq_norm")
        self.kv_norm = self._f32(block, "dkv_norm") if m.kv_from is None else None
        self.qp = _up(m.q_rank, 8)
        self.dim_p, self.vdim_p = _up(m.dim, 32), _up(m.vdim, 32)
        # columns: the heads' plain parts, then their rotated parts
        self.at_turned = m.heads * self.dim_p
        self.w_uq = self._zeros(self.qp, self.at_turned + m.heads * m.rot_pad)
        uq = block.uq.detach().view(m.heads, m.dim + m.rot_dim, m.q_rank)
        for name, at, padded, w in (
            ("uq_plain", 0, self.dim_p, uq[:, : m.dim]), ("uq_turned", self.at_turned, m.rot_pad, uq[:, m.dim :])
        ):
            view = self.w_uq[: m.q_rank, at : at + m.heads * padded].unflatten(1, (m.heads, padded))
            view = view[:, :, : w.shape[1]].permute(1, 2, 0)
            view.copy_(w)
            self._views[name] = view
        self.w_uk = self._zeros(m.heads, m.latent_pad, self.dim_p)
        self.w_uv = self._zeros(m.heads, self.vdim_p, m.latent_pad)
        self._place(block, "uv", self.w_uv[:, : m.vdim, : m.kv_rank])
        view = self.w_uk[:, : m.kv_rank, : m.dim].transpose(1, 2)
        self._place(block, "uk", view)
        self.w_o = self._zeros(m.heads * self.vdim_p, self.dp)
        self._place(block, "o", self.w_o.view(m.heads, self.vdim_p, self.dp)[:, : m.vdim, :d].permute(2, 0, 1))
        self.sink = self._f32(block, "sink")
        i = torch.arange(m.rot_turned // 2, dtype=torch.float64)
        quarters = m.rot_base ** (-2.0 * i / max(m.rot_turned, 1)) * (2.0 / math.pi)
        self.quarters = quarters.to(self.device)

    def _pack_forget(self, block):
        m = self.spec
        self.cols = self._columns(block, [
            ("q", m.heads, m.dim, m.dim), ("f", m.heads, m.dim, m.dim), ("v", m.heads, m.vdim, m.vdim),
        ])
        self.f_bias, self.lower = self._f32(block, "f_bias"), self._f32(block, "lower")
        self.head_norm = self._f32(block, "head_norm")
        self._pack_wide_o(block)

    def _pack_ssm(self, block):
        m = self.spec
        rows = block.in_proj.detach().split([m.inner, m.channels, m.heads])
        starts = [0, _up(m.inner, 8), _up(m.inner, 8) + _up(m.channels, 8)]
        self.w_in = self._zeros(self.dp, starts[2] + _up(m.heads, 8))
        for name, at, w in zip(("in_z", "in_conv", "in_dt"), starts, rows):
            self._views[name] = self.w_in[: self.d, at : at + len(w)].t()
            self._views[name].copy_(w)
        _, self.at_conv, self.at_dt = starts
        self.conv_w = block.conv.detach().float().t().contiguous()  # [taps, channels]
        self._views["conv"] = self.conv_w.t()
        self.conv_b = self._f32(block, "conv_bias")
        self.a_exp = self._f32(block, "A_log").exp()
        self.dt_bias, self.skip = self._f32(block, "dt_bias"), self._f32(block, "D")
        self.group_norm = self._f32(block, "group_norm")
        self._pack_wide_o(block)

    def _pack_wide_o(self, block):
        m = self.spec
        self.wide = _up(m.heads * m.vdim, 8)
        self.w_o = self._zeros(self.wide, self.dp)
        self._place(block, "o", self.w_o[: m.heads * m.vdim, : self.d].t())
        self.captures = self.hip.linear_decodes(m.dim if self.kind == "hgrn" else m.state, m.vdim)

    # ---------------------------------------------------------------- forward

    def forward_paged(self, x: torch.Tensor, batch, cache=None, state=None) -> torch.Tensor:
        """x [T, width] 32-bit, updated in place."""
        h = self.hip
        few = not self.f32 and x.shape[0] <= self.max_gemv_rows
        wide = few or self.f32  # 32-bit activations
        y = self._dense(h.residual_norm(x, None, None, self.norm1, self.d, self.eps, wide), self.w_in, few)
        y = self.run(y, batch, cache if state is None else state, few, wide)
        if self.mlp is None:
            self._add(x, y, self.w_o, few)
            return x
        n = self._add_and_norm(x, y, self.w_o, few, self.norm2)
        act = h.bias_xielu(self._dense(n, self.w_up, few, _EPI_RAW), self.b_up, *self.xielu)
        self._add(x, act, self.w_down, few, self.b_down)
        return x

    def _latent(self, y, batch, cache, few, wide):
        m, h, t = self.spec, self.hip, y.shape[0]
        cq, gate = h.latent_rows(
            y, self.at_q, self.q_norm, self.qp, wide, self.at_kv[0] if self.at_kv else -1, self.kv_norm, m.latent_pad,
            m.rot_dim, self.quarters, cache, self.at_g, m.heads, batch.pos, batch.owner, batch.tables, self.eps,
        )
        qs = self._dense(cq, self.w_uq, few)
        q = torch.empty(t, m.heads, m.latent_pad + m.rot_pad, dtype=cache.dtype, device=y.device)
        plain = qs[:, : self.at_turned].view(t, m.heads, self.dim_p)
        h.batched_linear(plain, self.w_uk, self.f32, q[:, :, : m.latent_pad])
        h.rotate_queries(qs, self.at_turned, m.rot_pad, self.quarters, batch.pos, q, m.latent_pad)
        run = batch.run_tokens(m.heads)
        lat = h.latent_attention(
            q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, batch.max_end, 0, m.scale, 0,
            m.latent_pad, self.sink, gate,
        )
        return h.batched_linear(lat, self.w_uv, wide).view(t, m.heads * self.vdim_p)

    def _forget(self, y, batch, state, few, wide):
        m, h, matrix = self.spec, self.hip, state["matrix"]
        sizes = (matrix, m.heads, m.dim, m.vdim, self.cols)
        if batch.decode_only and self.captures:
            y = h.forget_decode(
                y, self.f_bias, self.lower, self.head_norm, batch.pos, batch.slot, *sizes, self.wide, self.eps
            )
            return y
        o = h.forget_prefill(
            y, self.f_bias, self.lower, batch.tiles(CHUNK), batch.chunk_bounds(CHUNK), batch.pos, batch.owner,
            batch.slot, *sizes,
        )
        return h.group_norm(o, None, self.head_norm, m.heads, self.wide, wide, self.eps)

    def _ssm(self, y, batch, state, few, wide):
        m, h = self.spec, self.hip
        weights = (y, self.conv_w, self.conv_b, self.a_exp, self.dt_bias, self.skip)
        sizes = (state["matrix"], state["conv"], m.heads, m.groups, m.state, m.vdim, self.at_conv, self.at_dt)
        if batch.decode_only and self.captures:
            o = h.ssm_decode(*weights, batch.pos, batch.slot, *sizes)
        else:
            o = h.ssm_prefill(
                *weights, batch.tiles(CHUNK), batch.chunk_bounds(CHUNK), batch.pos, batch.owner, batch.slot, *sizes
            )
        return h.group_norm(o, y[:, : m.inner], self.group_norm, m.norm_groups, self.wide, wide, self.eps)
