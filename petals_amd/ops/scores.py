"""MI355X fast path of blocks whose attention and feed-forward read one norm, and whose
attention caps its scores, subtracts one softmax map from another or weighs keys by
sigmoids (models/zudarax).

Kernels: ops/csrc/{capped,paired,sigmoid}_attn.hip, prepare_rows.hip, prenorm.hip,
gemv.hip, in a library of their own (ops/build.py "scores").

Everything that reads the normed input is one product: queries, keys, values, output
gates and the feed-forward's inner rows. Attended values and activated inner rows lie
side by side, so that both sublayers' last products and their sum are one product too.
A layer is thus norm, product, preparation of rows (bias, convolution, norms, rotation,
cache, PolyNorm), attention, product, sum. Routes of few and many rows: ops/packed.py.
"""

from __future__ import annotations

import math

import torch

from petals_amd.ops import reference
from petals_amd.ops.packed import CHUNK, PackedBlock, attention_run
from petals_amd.ops.packed import round_up as _up


def hip():
    """The compiled kernels; on a GPU there is nothing else to fall back to."""
    from petals_amd.ops import _hip

    return _hip.first_loaded("scores")


class ScoresFastPath(PackedBlock):
    def __init__(self, block):
        super().__init__(block, hip())
        m, d = self.spec, self.d
        self.groups = block.groups
        self.norm1 = self._f32(block, "norm1")
        self.dk, self.dv = m.dim_pad, m.vdim_pad
        heads = {"q": (m.heads * m.maps, m.dim, self.dk), "k": (m.kv_heads * m.maps, m.dim, self.dk),
                 "v": (m.kv_heads, m.vdim, self.dv)}
        self.wide = m.heads * self.dv
        ff = 0 if self.mlp is None else self.mlp.ff
        ffp = _up(self.wide + ff, 64) - self.wide if ff else 0  # a sum of products that is cut in equal parts
        parts = [(name, *sizes) for name, sizes in heads.items()]
        if m.head_gate:
            parts.append(("g", m.heads, 1, 1))
        if ff:
            parts.append(("up", 1, ff, ffp))
        starts = dict(zip([p[0] for p in parts], self._columns(block, parts)))
        self.at_gate, self.at_up = starts.get("g"), starts.get("up", 0)
        self.bias = self._vector(block, "bias", heads) if m.bias else None
        self.qk_norm = self._vector(block, "norm", {n: heads[n] for n in "qk"}) if m.qk_norm else None
        self.conv_w = None
        if m.taps:  # [taps, columns]
            self.conv_w = torch.zeros(m.taps, m.columns, device=self.device)
            at = 0
            for name, (n, size, padded) in heads.items():
                view = self.conv_w[:, at : at + n * padded].unflatten(1, (n, padded))[:, :, :size].permute(1, 2, 0)
                self._place(block, f"{name}_conv", view)
                self._views[f"{name}_conv"] = view.reshape(n * size, m.taps)
                at += n * padded
        # the attended values' rows, then the feed-forward's
        self.w_out = self._zeros(self.wide + ffp, self.dp)
        o = self.w_out[: self.wide].view(m.heads, self.dv, self.dp)[:, : m.vdim, :d].permute(2, 0, 1)
        self._place(block, "o", o)
        self.poly = []
        if ff:
            self._place(block, "down", self.w_out[self.wide : self.wide + ff, :d].t())
            self.poly = self._f32(block, "act").tolist()
        freqs, self.turn_factor = reference.rotary_frequencies(m.rot.dims, m.rot.base, m.rot.yarn)
        self.quarters = (freqs * (2.0 / math.pi)).to(self.device)
        if m.sigmoid:
            self.pb = self._f32(block, "pb")
        if m.maps == 2:
            lams = [self._f32(block, n) for n in ("lq1", "lk1", "lq2", "lk2")]
            self.share = float(reference.differential_share(*lams, m.diff))
        self.captures = self.dk <= 256 and self.dv <= 256
        self._release(block)

    def _vector(self, block, kind, heads):
        """Per-channel vectors of the named projections, padded as their columns are."""
        out, at = torch.zeros(sum(n * padded for n, _, padded in heads.values()), device=self.device), 0
        for name, (n, size, padded) in heads.items():
            view = out[at : at + n * padded].view(n, padded)[:, :size]
            self._place(block, f"{name}_{kind}", view)
            self._views[f"{name}_{kind}"] = view.reshape(-1)
            at += n * padded
        return out

    # ---------------------------------------------------------------- forward

    def forward_paged(self, x: torch.Tensor, batch, cache: torch.Tensor, state=None) -> torch.Tensor:
        """x [T, width] 32-bit, updated in place; state: the convolution's inputs or None."""
        h, m = self.hip, self.spec
        few = not self.f32 and x.shape[0] <= self.max_gemv_rows
        wide = few or self.f32  # 32-bit activations
        n = h.residual_norm(x, None, None, self.norm1, self.d, self.eps, wide, 1.0, self.groups)
        y = self._dense(n, self.w_in, few)
        out = torch.empty(x.shape[0], self.w_out.shape[0], dtype=y.dtype, device=y.device)
        chunks = (None, None)
        if state is not None and not batch.decode_only:
            chunks = batch.tiles(CHUNK), batch.chunk_bounds(CHUNK)
        q = h.prepare_rows(
            y, cache, batch.pos, batch.owner, batch.tables, m.heads * m.maps, m.kv_heads * m.maps, self.dk, m.dim,
            m.kv_heads * self.dv, self.bias, self.conv_w, self.qk_norm, self.quarters, self.turn_factor, state,
            None if state is None else batch.slot, batch.decode_only, *chunks, self.poly, self.at_up,
            self.mlp.ff if self.poly else 0, out[:, self.wide :] if self.poly else None, self.eps,
        )
        self._attend(q, cache, batch, y, out)
        self._add(x, out, self.w_out, few)
        return x

    def _attend(self, q, cache, batch, y, out):
        """The heads' results into the first columns of `out`."""
        m, h, t = self.spec, self.hip, q.shape[0]
        run = attention_run(batch, m.heads, m.kv_heads)
        max_keys = min(batch.max_end, m.chunk) if m.chunk else batch.max_end
        rows = (
            cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, max_keys, m.kv_heads, self.dv, m.chunk,
            m.scale,
        )
        if m.maps == 2:
            gate = y[:, self.at_gate : self.at_gate + m.heads] if m.head_gate else None
            q = q.view(t, m.heads, 2, self.dk)
            h.paired_attention(q, *rows, self.share, 1.0 - m.diff, self.eps, m.vdim, gate, out)
        elif m.sigmoid:
            h.sigmoid_attention(q.view(t, m.heads, self.dk), *rows, self.pb, out)
        else:
            h.capped_attention(q.view(t, m.heads, self.dk), *rows, m.softcap, out)
