"""MI355X fast path of pre-norm blocks with windowed attention or a gated delta
rule and a dense feed-forward (models/lefulorn).

Kernels: ops/csrc/paged_attn.hip, delta.hip, prenorm.hip, gemv.hip, in a library
of their own (ops/build.py "hybrid").

Everything that reads the normed input is one product: queries, keys, values and
gate of attention; queries, keys, values, beta and the inner low-rank projections
of the delta rule. The delta rule has a kernel for batches of single tokens and a
chunked one for all others. Packing and routes: ops/packed.py.
"""

from __future__ import annotations

import torch

from petals_amd.models.lefulorn.config import KEY_PAD, VALUE_PAD
from petals_amd.ops import reference
from petals_amd.ops.packed import CHUNK, PackedBlock, attention_run
from petals_amd.ops.packed import round_up as _up

_EPI_RELU2_F32 = 6


def hip():
    """The compiled kernels; on a GPU there is nothing else to fall back to."""
    from petals_amd.ops import _hip

    return _hip.first_loaded("hybrid")


class HybridFastPath(PackedBlock):
    def __init__(self, block):
        super().__init__(block, hip())
        self.mix, self.carried = block.mix, block.config.carried_values
        self.norm1 = self._f32(block, "norm1")
        if block.delta:
            self._pack_delta(block)
        else:
            self._pack_attention(block)
        if self.mlp is not None:
            self.norm2 = self._f32(block, "norm2")
        self._finish(block)
        if self.mlp is not None:
            self.b_up_gemv = self.b_up.to(torch.bfloat16)

    def _pack_attention(self, block):
        a = self.spec
        self.dk, self.dv = _up(a.dim, KEY_PAD), _up(a.vdim, VALUE_PAD)
        _, at_k, at_v, self.at_gate = self._columns(block, [
            ("q", a.heads, a.dim, self.dk), ("k", a.kv_heads, a.dim, self.dk), ("v", a.kv_heads, a.vdim, self.dv),
            ("g", a.heads, a.vdim, self.dv),
        ])
        self.b_in = torch.zeros(self.at_gate, device=self.device)
        for name, at, heads, size, padded in (
            ("q_bias", 0, a.heads, a.dim, self.dk), ("k_bias", at_k, a.kv_heads, a.dim, self.dk),
            ("v_bias", at_v, a.kv_heads, a.vdim, self.dv),
        ):
            view = self.b_in[at : at + heads * padded].view(heads, padded)[:, :size]
            self._place(block, name, view)
            self._views[name] = view.reshape(-1)
        self.w_o = self._zeros(a.heads * self.dv, self.dp)
        self._place(block, "o", self.w_o.view(a.heads, self.dv, self.dp)[:, : a.vdim, : self.d].permute(2, 0, 1))
        self.sink = self._f32(block, "sink")
        self.slopes = reference.distance_slopes(a.heads, self.device)
        self.lam = self._f32(block, "vmix") if self.mix == "mix" else None
        self.captures = self.dk <= 256 and self.dv <= 256

    def _pack_delta(self, block):
        m = self.spec
        a_rank, g_rank = block.a1.shape[0], block.g1.shape[0]
        *self.cols, self.at_a1, self.at_g1 = self._columns(block, [
            ("q", m.kv_heads, m.dim, m.dim), ("k", m.kv_heads, m.dim, m.dim), ("v", m.heads, m.vdim, m.vdim),
            ("b", m.heads, 1, 1), ("a1", 1, a_rank, _up(a_rank, 8)), ("g1", 1, g_rank, _up(g_rank, 8)),
        ])
        self.w_a2 = self._zeros(m.heads * m.dim, _up(a_rank, 8))
        self.w_g2 = self._zeros(m.heads * m.vdim, _up(g_rank, 8))
        self._place(block, "a2", self.w_a2[:, :a_rank])
        self._place(block, "g2", self.w_g2[:, :g_rank])
        # [taps, channels]
        conv_w = torch.cat([getattr(block, f"{n}_conv").detach().float() for n in ("q", "k", "v")])
        self.conv_w = conv_w.t().contiguous()
        rows = [getattr(block, f"{n}_conv").shape[0] for n in ("q", "k", "v")]
        self._views.update(zip(("q_conv", "k_conv", "v_conv"), self.conv_w.t().split(rows)))
        self.a_exp = self._f32(block, "A_log").exp()
        self.dt_bias, self.o_norm = self._f32(block, "dt_bias"), self._f32(block, "o_norm")
        self.wide = _up(m.heads * m.vdim, 8)
        self.w_o = self._zeros(self.wide, self.dp)
        self._place(block, "o", self.w_o[: m.heads * m.vdim, : self.d].t())
        self.captures = self.hip.delta_decodes(m.dim, m.vdim)

    # ---------------------------------------------------------------- forward

    def forward_paged(self, x: torch.Tensor, batch, cache=None, state=None) -> torch.Tensor:
        """x [T, stream width] 32-bit, updated in place."""
        h = self.hip
        few = not self.f32 and x.shape[0] <= self.max_gemv_rows
        wide = few or self.f32  # 32-bit activations
        y = self._dense(h.residual_norm(x, None, None, self.norm1, self.d, self.eps, wide), self.w_in, few)
        y = self._attention(x, y, batch, cache, wide) if state is None else self._delta(y, batch, state, wide)
        if self.mlp is None:
            self._add(x, y, self.w_o, few)
            return x
        n = self._add_and_norm(x, y, self.w_o, few, self.norm2)
        if few:
            act = self._dense(n, self.w_up, few, _EPI_RELU2_F32, self.b_up_gemv)
        else:
            act = h.bias_relu2(n @ self.w_up, self.b_up)
        self._add(x, act, self.w_down, few, self.b_down)
        return x

    def _attention(self, x, y, batch, cache, wide):
        a, h = self.spec, self.hip
        first = x[:, self.d :] if self.mix else None
        q = h.attn_prepare(
            y, self.b_in, cache, batch.pos, batch.owner, batch.tables, a.heads, a.kv_heads, self.dk, self.dv,
            a.temp_coef, a.temp_every, first, self.lam, a.vdim,
        )
        run = attention_run(batch, a.heads, a.kv_heads)
        max_keys = min(batch.max_end, a.window) if a.window > 0 else batch.max_end
        return h.paged_attention(
            q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, max_keys, a.kv_heads, self.dv,
            a.window, a.scale, self.slopes, self.sink, y[:, self.at_gate : self.at_gate + a.heads * self.dv], wide,
        )

    def _delta(self, y, batch, state, wide):
        m, h = self.spec, self.hip
        delta, conv = state["delta"], state["conv"]
        sizes = (m.heads, m.kv_heads, m.dim, m.vdim, self.cols)
        if batch.decode_only and self.captures:
            return h.delta_decode(
                y, self.conv_w, self.w_a2, self.w_g2, self.at_a1, self.at_g1, self.a_exp, self.dt_bias, self.o_norm,
                batch.pos, batch.slot, delta, conv, *sizes, self.wide, self.eps,
            )
        a, gate = (
            self._outer(y[:, at : at + w.shape[1]], w) for at, w in ((self.at_a1, self.w_a2), (self.at_g1, self.w_g2))
        )
        o = h.delta_prefill(
            y, a, self.conv_w, self.a_exp, self.dt_bias, batch.tiles(CHUNK), batch.chunk_bounds(CHUNK), batch.pos,
            batch.owner, batch.slot, delta, conv, *sizes,
        )
        return h.delta_norm(o, gate, self.o_norm, m.heads, self.wide, wide, self.eps)

    def _outer(self, x, w):
        """x [T, rank] @ w [n, rank].T with a 32-bit result."""
        if self.f32:
            return x @ w.t()
        return self.hip.batched_linear(x.unsqueeze(1), w.unsqueeze(0), True).squeeze(1)
