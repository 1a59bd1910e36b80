"""Zudarax against its plain oracle (tests/zudarax_oracle.py): mechanisms alone, and
whole models through the span engine that serves them - prompts, portions, decoding,
mixed batches, pages and state slots used again - on the CPU path and, marked gpu, on
the HIP kernels in float32 and bfloat16."""

import copy
import json
import math
import random

import pytest
import torch

import zudarax_oracle as oracle
from petals_amd.models.config_base import load_model_config
from petals_amd.models.zudarax.config import YarnSpec
from petals_amd.ops import reference
from petals_amd.server.from_pretrained import load_pretrained_block
from petals_amd.server.memory_cache import AllocationFailed
from petals_amd.server.paged_cache import PAGE_SIZE, PagedBatch
from petals_amd.server.span_engine import SpanEngine, StepEntry

PATHS = [
    ("cpu", "float32"),
    pytest.param(("cuda", "float32"), marks=pytest.mark.gpu),
    pytest.param(("cuda", "bfloat16"), marks=pytest.mark.gpu),
]
TOLERANCE = {"float32": 2e-4, "bfloat16": 5e-2}  # of the residual's own size
F64 = torch.float64

C, P, S = oracle.capped_layer, oracle.paired_layer, oracle.sigmoid_layer
SHAPES = {
    # every kind of layer with and without a feed-forward, one kind twice in a row
    "mixed": [
        S(heads=4, kv_heads=2, dim=20, vdim=12, rot=16, ff=None), C(heads=6, kv_heads=2, dim=16, vdim=20, ff=40), P(ff=36),
        P(heads=3, kv_heads=3, dim=24, vdim=8, rot=24, diff=0.3), C(size=17, conv=2, rot=16, base=40.0, ff=None), S(conv=5),
    ],
    # everything that can be one is one
    "ones": [
        C(heads=1, kv_heads=1, dim=2, vdim=1, conv=1, size=1, rot=2, ff=1),
        P(heads=1, kv_heads=1, dim=2, vdim=1, rot=2, ff=1), S(heads=1, kv_heads=1, dim=2, vdim=1, conv=1, rot=2, ff=1),
    ],
    # equal sizes everywhere
    "equal": [
        C(heads=32, kv_heads=32, dim=32, vdim=32, size=32, rot=32, ff=32, conv=4),
        P(heads=32, kv_heads=32, dim=32, vdim=32, rot=32, ff=32), S(heads=32, kv_heads=32, dim=32, vdim=32, rot=32, ff=32),
    ],
    # head counts and sizes that are no multiple of anything, more heads to a key than a tile has rows
    "wide": [
        C(heads=18, kv_heads=1, dim=33, vdim=65, conv=7, size=100, rot=10, ff=77), P(heads=70, kv_heads=1, dim=9, vdim=35, rot=8),
        S(heads=34, kv_heads=2, dim=72, vdim=40, rot=66), P(heads=6, kv_heads=2, dim=50, vdim=133, rot=44, ff=131),
        C(heads=5, kv_heads=5, dim=130, vdim=40, rot=0, size=64),
    ],
    # beyond the tiled kernels' sizes
    "long_heads": [
        C(heads=2, kv_heads=1, dim=24, vdim=270), P(heads=2, kv_heads=2, dim=260, vdim=300, rot=100), S(heads=2, kv_heads=1, dim=270, vdim=20),
    ],
    "no_state": [P(), P(heads=2, kv_heads=1, ff=24)],
}


class Model:
    """A random model served by a SpanEngine, and its oracle. (A norm over few values that
    happen to be small amplifies bf16 rounding without bound if eps is tiny.)"""

    def __init__(self, tmp_path, layers, path=("cpu", "float32"), *, width=40, vocab=97, tokens=1024, seed=0, edit=None,
                 eps=1e-2, groups=2, sequences=None):
        self.device, self.dtype = path
        self.raw = oracle.config_dict(vocab=vocab, width=width, layers=layers, eps=eps, groups=groups)
        self.weights = oracle.random_model(self.raw, seed)
        if edit is not None:
            edit(self.weights)
        self.dir = str(tmp_path / "model")
        oracle.save_model(self.dir, self.raw, self.weights)
        self.config = load_model_config(self.dir)
        dtype = getattr(torch, self.dtype)
        blocks = {
            i: load_pretrained_block(self.dir, self.config, i, torch_dtype=dtype, device=self.device)
            for i in range(self.config.num_blocks)
        }
        pool = SpanEngine.pool_for(
            list(blocks.values()), tokens, dtype=dtype, device=self.device, max_sequences=sequences
        )
        self.engine = SpanEngine(blocks, pool, max_length=tokens)
        self.uids = tuple(blocks)

    def embed(self, ids):
        return self.weights["embed"][torch.as_tensor(ids)].float().to(self.device)

    def residual(self, y):
        return y.detach().double().cpu()

    def expected(self, ids, faults=()):
        res = []
        oracle.run(self.raw, self.weights, ids, residuals=res, faults=frozenset(faults))
        return res[-1]

    def run(self, ids, cuts=None, sequence=None):
        """The residual of one request, its tokens cut into steps of the given sizes."""
        seq = sequence or self.engine.pool.open()
        out, at = [], 0
        for n in cuts or [len(ids)]:
            (y,) = self.engine.step(self.uids, [StepEntry(seq, self.embed(ids[at : at + n]), at)])
            assert torch.is_tensor(y), y
            out.append(y)
            at += n
        assert at == len(ids)
        if sequence is None:
            seq.close()
        return self.residual(torch.cat(out))

    def errors(self, got, want):
        """RMS difference at each position, relative to the residual's RMS."""
        return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()

    def error(self, got, want):
        return float(self.errors(got, want).max())

    def check(self, got, want, slack=1.0):
        """All but a few positions within the tolerance, and none far from it."""
        e, limit = self.errors(got, want), slack * TOLERANCE[self.dtype]
        assert float(e.max()) < 2.5 * limit and int((e > limit).sum()) <= 0.02 * len(e) + 1, e.topk(min(5, len(e)))


def ids_of(n, vocab=97, seed=1):
    return random.Random(seed).choices(range(vocab), k=n)


# ------------------------------------------------------------- mechanisms


@pytest.mark.parametrize("n,dims", [(8, 8), (2, 2), (10, 6), (5, 0)])
@pytest.mark.parametrize("yarn", [None, (6.0, 90, 10.0, 0.5), (3.0, 1000, 2.0, 2.0), (1.0, 64, 32.0, 1.0), (16.0, 4, 9.0, 3.0)])
def test_rotation_with_scaled_frequencies(n, dims, yarn):
    rot = {"dims": dims, "base": 70.0}
    if yarn is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    x = torch.randn(70, 3, n, dtype=F64)
    freqs, factor = reference.rotary_frequencies(dims, 70.0, yarn and YarnSpec(*yarn))
    got = reference.rotate_pairs(x, torch.arange(70)[:, None], freqs, factor)
    assert (got - oracle.rotate(x, torch.arange(70), rot)).abs().max() < 1e-6
    want, grows = oracle.frequencies(rot)
    assert factor == (grows if dims else 1.0) and torch.allclose(freqs, torch.tensor(want, dtype=F64), rtol=1e-12)


def test_scaling_divides_slow_pairs_only():
    rot = {"dims": 32, "base": 10000.0, "scaling": {"factor": 8.0, "original": 700, "fast": 20.0, "slow": 1.5}}
    plain, scaled = (torch.tensor(oracle.frequencies({**rot, "scaling": s})[0]) for s in (None, rot["scaling"]))
    ratio = plain / scaled
    assert ratio[0] == 1.0 and torch.isclose(ratio[-1], torch.tensor(8.0)) and (ratio.diff() >= 0).all()
    assert ((ratio > 1.01) & (ratio < 7.9)).any()


@pytest.mark.parametrize("taps", [1, 2, 3, 6])
def test_short_convolution_and_its_last_inputs(taps):
    u, w = torch.randn(20, 5, dtype=F64), torch.randn(5, taps, dtype=F64)
    want = oracle.short_conv(u, w)
    padded = torch.cat([torch.zeros(taps - 1, 5, dtype=F64), u])
    assert (reference.short_conv(padded[None], w)[0] - want).abs().max() < 1e-12
    half = reference.short_conv(padded[None, 10:], w)[0]  # the second half from the last inputs of the first
    assert (half - want[10:]).abs().max() < 1e-12


def dense_inputs(s, heads, kv, dim, vdim, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(s, heads, dim, generator=g), torch.randn(s, kv, dim, generator=g), torch.randn(s, kv, vdim, generator=g)


@pytest.mark.parametrize("chunk", [0, 1, 7, 40])
@pytest.mark.parametrize("kind", ["softmax", "capped", "sigmoid"])
def test_scored_attention(kind, chunk):
    q, k, v = dense_inputs(40, 6, 2, 8, 5)
    bias = torch.linspace(-3, 1, 6)
    pos = torch.arange(40)
    seen = reference.visible(pos, pos, chunk=chunk)
    got = reference.scored_attention(
        q, k, v, seen, scale=0.6, softcap=1.5 if kind == "capped" else 0.0, sigmoid_bias=bias if kind == "sigmoid" else None
    )
    mask = oracle.same_chunk(40, chunk) if chunk else oracle.causal(40)
    assert torch.equal(mask, seen)
    for h in range(6):
        score = q[:, h].double() @ k[:, h // 3].double().T * 0.6
        if kind == "capped":
            score = oracle.cap(score, 1.5)
        p = oracle.sigmoid_weights(score, mask, bias[h].double()) if kind == "sigmoid" else oracle.softmax_weights(score, mask)
        assert (got[:, h] - p @ v[:, h // 3].double()).abs().max() < 1e-5


def test_share_of_the_second_map():
    w = {n: 0.3 * torch.randn(12, dtype=F64) for n in ("lq1", "lk1", "lq2", "lk2")}
    got = reference.differential_share(*(w[n] for n in ("lq1", "lk1", "lq2", "lk2")), 0.4)
    assert abs(float(got) - float(oracle.share_of_second_map(w, 0.4))) < 1e-5


@pytest.mark.parametrize("scale", [1e-4, 1.0, 300.0])
def test_poly_norm(scale):
    z, act = scale * torch.randn(9, 50), torch.tensor([0.7, -0.4, 1.2, 0.3])
    want = oracle.poly_norm(z.double(), act.double(), 1e-6)
    assert (reference.poly_norm(z, act, 1e-6).double() - want).abs().max() < 1e-4


@pytest.mark.parametrize("groups", [1, 2, 6])
def test_norm_in_groups(groups):
    x, w = torch.randn(7, 12), torch.randn(12)
    want = oracle.group_norm(x.double(), w.double(), groups, 1e-3)
    assert (reference.group_rms_norm(x, w, groups, 1e-3).double() - want).abs().max() < 1e-5


def test_config_reads_every_layer_and_rejects_nonsense(tmp_path):
    raw = oracle.config_dict(layers=SHAPES["mixed"], width=24, eps=3e-5, groups=3)
    oracle.save_model(str(tmp_path), raw, {"x": torch.zeros(1)})
    c = load_model_config(str(tmp_path))
    assert (c.num_blocks, c.hidden_size, c.layer_norm_eps, c.norm_groups, c.model_type) == (6, 24, 3e-5, 3, "zudarax")
    m = c.spec(4).mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.taps, m.chunk, m.softcap, m.rot.base) == (4, 2, 16, 12, 2, 17, 3.0, 40.0)
    assert m.bias and m.qk_norm and m.maps == 1 and not m.sigmoid and not m.head_gate and c.spec(4).mlp is None
    m = c.spec(3).mixer
    assert (m.maps, m.diff, m.head_gate, m.taps, m.chunk, m.softcap, m.bias) == (2, 0.3, True, 0, 0, 0.0, False)
    m = c.spec(5).mixer
    assert m.sigmoid and m.taps == 5 and m.rot.yarn == YarnSpec(6.0, 90, 10.0, 0.5) and c.spec(5).mlp.ff == 30
    assert c.cache_values_per_token(3) == 3 * (2 * 32 + 16) and c.cache_values_per_token(0) == 2 * (32 + 16)
    assert c.state_shapes(3) == {} and c.state_shapes(0) == {"conv": (4, 6 * 32 + 2 * 16)} and not c.rewindable

    def broken(change):
        d = copy.deepcopy(raw)
        change(d)
        (tmp_path / "config.json").write_text(json.dumps(d))
        with pytest.raises((ValueError, KeyError)):
            load_model_config(str(tmp_path))

    broken(lambda d: d["layers"][0].update(type="attention_4"))
    broken(lambda d: d["layers"][1]["mixer"].update(kv_heads=4))
    broken(lambda d: d["layers"][1]["mixer"].update(conv=0))
    broken(lambda d: d["layers"][1]["mixer"]["mask"].update(size=0))
    broken(lambda d: d["layers"][1]["mixer"].pop("softcap"))
    broken(lambda d: d["layers"][2]["mixer"].pop("diff"))
    broken(lambda d: d["layers"][2]["mixer"]["rot"].update(dims=5))
    broken(lambda d: d["layers"][2]["mixer"]["rot"].update(dims=14))
    broken(lambda d: d["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0))
    broken(lambda d: d["layers"][1]["mlp"].update(kind="experts"))
    broken(lambda d: d["layers"][1]["mixer"].update(heads=2.5))
    broken(lambda d: d["norm"].update(groups=5))


def test_loader_refuses_incomplete_checkpoints(tmp_path):
    raw = oracle.config_dict(layers=SHAPES["mixed"])
    for name, change in (("l0.mix.pb", None), ("l1.mix.k.norm", None), ("l1.mix.q.b", lambda t: t[1:]),
                         ("l2.mix.lq2", None), ("l3.mix.k", lambda t: t[: len(t) // 2]),
                         ("l4.mix.v.conv", lambda t: t[:, 1:]), ("l5.mlp.act", lambda t: t[:3])):
        weights = oracle.random_model(raw)
        if change is None:
            del weights[name]
        else:
            weights[name] = change(weights[name]).contiguous()
        oracle.save_model(str(tmp_path), raw, weights)
        with pytest.raises((KeyError, ValueError), match=name.split(".", 1)[1]):
            load_pretrained_block(str(tmp_path), load_model_config(str(tmp_path)), int(name[1]), torch_dtype=torch.float32)


# ----------------------------------------------------------------- models


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_prompt_matches_oracle(tmp_path, shape, path):
    m = Model(tmp_path, SHAPES[shape], path)
    ids = ids_of(110)
    want = m.expected(ids)
    m.check(m.run(ids), want)
    m.check(m.run(ids, [90] + [1] * 20), want)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("width,vocab,eps,groups", [(8, 11, 1e-6, 1), (131, 40, 0.5, 131), (132, 60, 1e-4, 11), (256, 300, 0.3, 4)])
def test_other_widths_and_constants(tmp_path, width, vocab, eps, groups, path):
    m = Model(tmp_path, SHAPES["mixed"], path, width=width, vocab=vocab, eps=eps, seed=3, groups=groups)
    ids = ids_of(90, vocab)
    want = m.expected(ids)
    slack = 2.0 if width == 8 or groups > 4 else 1.0  # a norm over a handful of values amplifies rounding
    m.check(m.run(ids), want, slack)
    m.check(m.run(ids, [70] + [1] * 20), want, slack)


@pytest.mark.parametrize("path", PATHS[:2])
def test_every_fault_would_show(tmp_path, path):
    """The inputs of these tests tell each planted mistake from the design."""
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = ids_of(110)
    got = m.run(ids)
    for fault in (
        "one_norm_group", "no_conv", "conv_one_less", "conv_forgets", "conv_reversed", "no_yarn", "no_yarn_factor",
        "no_rotation", "rotate_neighbours", "forgets_far", "chunk_slides", "chunk_one_off", "no_score_bias", "normalized",
        "no_bias", "norm_per_head", "no_qk_norm", "no_cap", "lambda_constant", "maps_outside", "one_map", "no_map_norm",
        "no_map_factor", "no_gate", "no_constant", "powers_of_norm", "in_turn",
    ):
        assert m.error(got, m.expected(ids, [fault])) > 20 * TOLERANCE[m.dtype], fault


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("cuts", [
    [1] * 140, [100] + [1] * 40, [2] * 70, [2, 3, 64, 1, 63, 2, 5], [64, 64, 12], [63, 65, 12], [9, 131], [139, 1],
    [16] * 8 + [12], [17] * 8 + [4], [3, 1] * 35, [50, 50, 40],
], ids=lambda c: "-".join(map(str, c[:4])))
def test_portions_and_decoding_match_the_whole(tmp_path, cuts, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = ids_of(140)
    m.check(m.run(ids, cuts), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_long_decoding(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path, seed=5)
    ids = ids_of(330)
    m.check(m.run(ids, [10] + [1] * 320), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_unequal_requests_in_one_batch(tmp_path, path):
    """Prompts' portions beside decoded tokens, requests joining, pausing and
    leaving; every position equals the request alone."""
    m = Model(tmp_path, SHAPES["mixed"], path, sequences=11)
    plans = {
        "a": [1] * 60, "b": [37, 2, 1, 64, 1, 3], "c": [5, 1, 1, 90], "d": [1, 1, 70, 2], "e": [130], "f": [2] * 20,
        "g": [1] * 12, "h": [3] + [1] * 30, "i": [1] * 40, "j": [1] * 40, "k": [66] + [1] * 9,
    }
    ids = {k: ids_of(sum(p), seed=ord(k)) for k, p in plans.items()}
    rng = random.Random(0)
    seqs, at, outs = {}, {k: 0 for k in plans}, {k: [] for k in plans}
    left = {k: list(p) for k, p in plans.items()}
    while any(left.values()):
        live = [k for k in plans if left[k]]
        now = [k for k in live if rng.random() < 0.8][:10] or live[:1]
        rng.shuffle(now)
        entries = []
        for k in now:
            n = left[k].pop(0)
            if k not in seqs:
                seqs[k] = m.engine.pool.open()
            entries.append(StepEntry(seqs[k], m.embed(ids[k][at[k] : at[k] + n]), at[k]))
            at[k] += n
        for k, y in zip(now, m.engine.step(m.uids, entries)):
            outs[k].append(y)
            if not left[k]:
                seqs[k].close()
    for k in plans:
        m.check(m.residual(torch.cat(outs[k])), m.expected(ids[k]))
    assert m.engine.pool.free_pages == m.engine.pool.num_pages and len(m.engine.pool._free_slots) == 11


@pytest.mark.parametrize("path", PATHS)
def test_pages_and_slots_are_used_again_in_any_order(tmp_path, path):
    """A pool of five pages and two slots, scrambled and full of other requests' state."""
    m = Model(tmp_path, SHAPES["mixed"], path, tokens=5 * PAGE_SIZE, sequences=2)
    pool = m.engine.pool
    for round_, n in enumerate((320, 200, 129, 64, 65)):
        m.run(ids_of(n, seed=round_ + 50))
        random.Random(round_).shuffle(pool._free)
        pool._free_slots.reverse()
        ids = ids_of(200, seed=round_)
        m.check(m.run(ids, [100, 27, 1, 1, 71] if round_ % 2 else [1, 1, 127, 71]), m.expected(ids))
    a, b = pool.open(), pool.open()
    with pytest.raises(AllocationFailed, match="slots"):
        pool.open()
    m.run(ids_of(190), sequence=a)
    with pytest.raises(AssertionError, match="pages needed"):
        m.run(ids_of(190), sequence=b)
    a.close()
    ids = ids_of(190)
    m.check(m.run(ids, sequence=b), m.expected(ids))


QUERY, KEY = 90, 91


def standing_out(layer):
    """Weights of a one-layer model under which token QUERY scores far higher on token KEY
    than on any other, through a dimension that is not rotated."""
    m, kind = layer["mixer"], layer["type"]
    at = m["rot"]["dims"]

    def edit(w):
        p = "l0.mix."
        w["embed"][:, :2] = 0
        w["embed"][QUERY, 0] = 6.0
        w["embed"][KEY, 1] = 6.0
        w["l0.norm1"][:] = 1.0
        w[p + "o"] *= 4
        for n, source in (("q", 0), ("k", 1)):
            w[p + n][:] = 0
            rows = w[p + n].view(-1, m["dim"], w[p + n].shape[1])
            if kind == "attention":  # normed to the root of dim afterwards
                rows[:, at, source] = 1.0
                w[p + n + ".b"][:] = 0
                w[p + n + ".norm"][:] = 1.0
            elif kind == "attention_2":
                rows[::2, at, source] = 1.6
            else:
                rows[:, at, source] = 1.6
        for n in "qkv" if kind != "attention_2" else "":  # the convolution passes its last input
            w[p + n + ".conv"][:] = 0
            w[p + n + ".conv"][:, -1] = 1.0
        if kind == "attention_3":
            w[p + "pb"][:] = -9.0

    return edit


def far(kind, heads, kv_heads, size=150):
    if kind == "attention":
        return C(heads=heads, kv_heads=kv_heads, dim=24, vdim=16, rot=2, size=size, scale=0.5, softcap=30.0, ff=None)
    if kind == "attention_2":
        return P(heads=heads, kv_heads=kv_heads, dim=16, vdim=16, rot=2, scale=0.3, ff=None)
    return S(heads=heads, kv_heads=kv_heads, dim=16, vdim=16, rot=2, scale=0.4, ff=None)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("kind", ["attention_2", "attention_3"])
@pytest.mark.parametrize("heads,kv_heads", [(2, 1), (18, 1), (3, 3)])
def test_far_keys_and_page_borders(tmp_path, path, kind, heads, kv_heads):
    """One key among hundreds, at and around the borders of pages and tiles."""
    layer = far(kind, heads, kv_heads)
    m = Model(tmp_path, [layer], path, edit=standing_out(layer))
    n = 520
    for key in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 447, 448, 511, 518)[:: 1 if heads == 2 else 4]:
        ids = ids_of(n, vocab=80)
        ids[key], ids[n - 1] = KEY, QUERY
        want = m.expected(ids)
        assert m.error(want[-1:], m.expected(ids[:key] + [5] + ids[key + 1 :])[-1:]) > 0.1  # without that key
        for cuts in ([n], [n - 1, 1], [300, 219, 1]):
            m.check(m.run(ids, cuts), want)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("size", [1, 2, 32, 50, 64, 128, 150, 511])
def test_keys_just_inside_and_just_outside_a_chunk(tmp_path, path, size):
    """A query's chunk begins at a multiple of its size, wherever pages, tiles and portions end."""
    layer = far("attention", 4, 2, size=size)
    m = Model(tmp_path, [layer], path, edit=standing_out(layer))
    n = 512
    edge = (n - 1) // size * size
    for at in sorted({edge, min(edge + size // 2, n - 1), n - 1}):  # where the query stands
        for key in sorted({edge - 1, edge, at - 1} & set(range(at))):
            ids = ids_of(n, vocab=80)
            ids[key], ids[at] = KEY, QUERY
            want, without = m.expected(ids), m.expected(ids[:key] + [5] + ids[key + 1 :])
            change = m.error(want[at : at + 1], without[at : at + 1])
            assert change > 0.1 if key >= edge else change < 1e-9
            for cuts in ([n], [at, n - at], [at, 1, n - 1 - at], [max(1, at - 1), 2, n - at - 1], [key, n - key]):
                cuts = [c for c in cuts if c > 0]
                m.check(m.run(ids, cuts + [n - sum(cuts)] if sum(cuts) < n else cuts), want)


@pytest.mark.parametrize("path", PATHS)
def test_chunk_edges_in_decoding(tmp_path, path):
    layer = far("attention", 2, 1, size=70)
    m = Model(tmp_path, [layer], path, edit=standing_out(layer))
    ids = ids_of(230, vocab=80)
    for i in range(60, 230):  # a key at each chunk's first and last position, queries elsewhere
        ids[i] = KEY if i % 70 in (0, 69) else QUERY if i % 3 else ids[i]
    want = m.expected(ids)
    assert m.error(want, m.expected(ids, ["chunk_one_off"])) > 0.1
    m.check(m.run(ids, [60] + [1] * 170), want)
    m.check(m.run(ids, [2] * 115), want)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("taps", [1, 2, 4, 6])
def test_convolution_reaches_over_steps(tmp_path, path, taps):
    """The first tap alone: what a token attends with is an input some tokens ago, which an
    earlier step, another page or nothing ahead of the sequence has left."""

    def edit(w):
        for name, t in w.items():
            if name.endswith(".conv"):
                t[:, 1:] = 0

    layers = [C(conv=taps, size=20, ff=None), S(conv=taps, ff=None)]
    m = Model(tmp_path, layers, path, edit=edit)
    ids = ids_of(75)
    want = m.expected(ids)
    for cuts in ([75], [1] * 75, [2] * 37 + [1], [3, 1, 1, 2] * 10 + [5], [64, 11], [66, 9], [5] * 15, [40, 2, 1, 1, 20, 11]):
        m.check(m.run(ids, cuts), want)


@pytest.mark.parametrize("path", PATHS)
def test_scores_far_beyond_the_cap_and_the_sigmoid(tmp_path, path):
    """Weights stay finite where a tanh or a sigmoid is flat, and differ where they are not."""

    def edit(w):
        w["l0.mix.q.norm"] *= 6
        w["l1.mix.pb"][:] = torch.tensor([-90.0, 90.0, 0.0, -3.0])
        w["l1.mix.q"] *= 8

    m = Model(tmp_path, [C(heads=4, softcap=0.5, ff=None), S(heads=4, kv_heads=2, ff=None)], path, edit=edit)
    ids = ids_of(100)
    want = m.expected(ids)
    assert torch.isfinite(want).all() and m.error(want, m.expected(ids, ["no_cap"])) > 0.1
    m.check(m.run(ids), want)
    m.check(m.run(ids, [60] + [1] * 40), want)


@pytest.mark.parametrize("path", PATHS)
def test_first_tokens(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    for n in (1, 2, 3, 4, 5, 6):
        ids = ids_of(n, seed=n)
        m.check(m.run(ids), m.expected(ids))
        m.check(m.run(ids, [1] * n), m.expected(ids))
        if n > 2:
            m.check(m.run(ids, [2] + [1] * (n - 2)), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_rollback_only_to_the_start(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    seq = m.engine.pool.open()
    m.run(ids_of(70, seed=3), sequence=seq)
    (y,) = m.engine.step(m.uids, [StepEntry(seq, m.embed([1]), 60)])
    assert isinstance(y, ValueError) and "replay from 0" in str(y)
    ids = ids_of(90)
    m.check(m.run(ids, [89, 1], sequence=seq), m.expected(ids))
    m.check(m.run(ids, [1] * 90, sequence=seq), m.expected(ids))
    seq.close()
    # without a convolution the pages roll back as those of other families
    m = Model(tmp_path, SHAPES["no_state"], path)
    assert m.config.rewindable
    seq = m.engine.pool.open()
    ids = ids_of(100)
    m.run(ids[:80] + ids_of(20, seed=8), sequence=seq)
    (y,) = m.engine.step(m.uids, [StepEntry(seq, m.embed(ids[80:]), 80)])
    m.check(m.residual(y), m.expected(ids)[80:])


@pytest.mark.parametrize("path", PATHS)
def test_beam_reorder_copies_state(tmp_path, path):
    """Two of three hypotheses continue the second one, the third goes on with the first."""
    m = Model(tmp_path, SHAPES["mixed"], path)
    pool = m.engine.pool
    heads = [ids_of(70, seed=s) for s in (1, 2, 3)]
    seqs = [pool.open() for _ in heads]
    for s, t in zip(seqs, heads):
        m.run(t, sequence=s)
    pool.reorder(seqs, [1, 1, 0])
    tails = [ids_of(30, seed=s) for s in (4, 5, 6)]
    outs = [[], [], []]
    for i in range(30):
        ys = m.engine.step(m.uids, [StepEntry(s, m.embed([t[i]]), 70 + i) for s, t in zip(seqs, tails)])
        for o, y in zip(outs, ys):
            o.append(y)
    for o, parent, t in zip(outs, (1, 1, 0), tails):
        m.check(m.residual(torch.cat(o)), m.expected(heads[parent] + t)[70:])
    for s in seqs:
        s.close()
    assert pool.free_pages == pool.num_pages and not any(pool._refs)


@pytest.mark.parametrize("path", PATHS)
def test_long_steps_are_cut(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    m.engine.max_step_tokens = 50
    ids = [ids_of(130, seed=1), ids_of(20, seed=2), ids_of(45, seed=3)]
    seqs = [m.engine.pool.open() for _ in ids]
    xs = [m.embed(t) for t in ids]
    before = [x.clone() for x in xs]
    ys = m.engine.step(m.uids, [StepEntry(s, x, 0) for s, x in zip(seqs, xs)])
    for y, t, x, b in zip(ys, ids, xs, before):
        m.check(m.residual(y), m.expected(t))
        assert torch.equal(x, b)  # inputs are not touched


@pytest.mark.parametrize("path", PATHS)
def test_many_rows_in_a_step(tmp_path, path):
    """More rows than the kernels' small layouts take, in several sequences, and sums long
    enough to be cut in parts."""
    m = Model(tmp_path, [C(ff=2100), P(ff=1000), S(conv=3)], path, tokens=1600)
    ids = [ids_of(n, seed=n) for n in (601, 3, 210)]
    seqs = [m.engine.pool.open() for _ in ids]
    ys = m.engine.step(m.uids, [StepEntry(s, m.embed(t), 0) for s, t in zip(seqs, ids)])
    for y, t in zip(ys, ids):
        m.check(m.residual(y), m.expected(t))


@pytest.mark.parametrize("path", PATHS[:2])
def test_chain_in_two_engines(tmp_path, path):
    """The span cut between any two blocks, as two servers would run it."""
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = ids_of(60)
    assert m.config.valid_cuts() is None
    for cut in (1, 3, 5):
        engines = [
            SpanEngine(
                {u: m.engine.blocks[u] for u in part},
                SpanEngine.pool_for([m.engine.blocks[u] for u in part], 128, dtype=getattr(torch, m.dtype), device=m.device),
                max_length=128,
            )
            for part in (m.uids[:cut], m.uids[cut:])
        ]
        seqs, at, out = [e.pool.open() for e in engines], 0, []
        for n in (50, 1, 9):
            x = m.embed(ids[at : at + n])
            for e, s in zip(engines, seqs):
                (x,) = e.step(tuple(e.blocks), [StepEntry(s, x, at)])
            out.append(x)
            at += n
        m.check(m.residual(torch.cat(out)), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_stateless_forward_equals_the_cached_one(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = [ids_of(75, seed=1), ids_of(75, seed=2)]
    x = torch.stack([m.embed(t) for t in ids])
    cached, plain = m.engine.forward(m.uids, x), x
    for uid in m.uids:
        plain = m.engine.blocks[uid](plain)
    for i, t in enumerate(ids):
        m.check(m.residual(cached[i]), m.expected(t))
        m.check(m.residual(plain[i]), m.expected(t))


# --------------------------------------------------------- kernels, one by one


def max_error(got, want):
    return float((got.double().cpu() - want).abs().max() / want.abs().max())


@pytest.mark.gpu
@pytest.mark.parametrize("kind", ["capped", "paired", "sigmoid"])
@pytest.mark.parametrize("heads,kv_heads,dk,dv,dtype", [
    (1, 1, 32, 16, "bfloat16"), (8, 2, 64, 48, "bfloat16"), (17, 1, 128, 64, "bfloat16"), (6, 6, 96, 128, "bfloat16"),
    (4, 2, 224, 256, "bfloat16"), (66, 1, 32, 32, "bfloat16"), (2, 1, 256, 80, "bfloat16"), (3, 1, 288, 32, "bfloat16"),
    (2, 2, 32, 272, "bfloat16"), (6, 2, 64, 48, "float32"), (1, 1, 288, 304, "float32"),
])
def test_attention_kernels(kind, heads, kv_heads, dk, dv, dtype):
    """Every key split and row layout agrees with the dense computation, on scattered
    pages, over everything and over chunks, into a part of wider rows."""
    from petals_amd.ops import scores

    torch.manual_seed(0)
    hip, dt, maps, group = scores.hip(), getattr(torch, dtype), 2 if kind == "paired" else 1, heads // kv_heads
    vdim = dv - 3 if kind == "paired" else dv
    scale, wide = 1.5 * dk**-0.5, kv_heads * maps * dk
    cache = torch.randn(9, PAGE_SIZE, wide + kv_heads * dv, device="cuda").to(dt)
    cache[..., wide:].unflatten(-1, (kv_heads, dv))[..., vdim:] = 0
    bias = torch.linspace(-5, 2, heads, device="cuda")
    for starts, lens in (([0, 130, 63], [40, 1, 70]), ([0, 130, 63], [1, 1, 1])):
        pages = [[3], [5, 0, 7], [8, 1, 2]]
        batch = PagedBatch(pages, starts, lens, torch.device("cuda"))
        q = torch.randn(batch.tokens, heads, maps, dk, device="cuda").to(dt)
        gate = torch.randn(batch.tokens, heads + 3, device="cuda").to(dt)[:, 2 : 2 + heads]
        run = batch.run_tokens(group)
        for chunk in (0, 50):
            want = torch.empty(batch.tokens, heads, dv, dtype=F64)
            for (lo, hi), p, s in zip(batch.row_ranges(), pages, starts):
                rows = cache[p].reshape(-1, cache.shape[-1])[: s + hi - lo].double().cpu()
                keys, values = rows[:, :wide].unflatten(1, (kv_heads, maps, dk)), rows[:, wide:].unflatten(1, (kv_heads, dv))
                seen = (oracle.same_chunk(len(rows), chunk) if chunk else oracle.causal(len(rows)))[s:]
                for n in range(heads):
                    score = [q[lo:hi, n, u].double().cpu() @ keys[:, n // group, u].T * scale for u in range(maps)]
                    if kind == "sigmoid":
                        o = oracle.sigmoid_weights(score[0], seen, bias[n].double().cpu()) @ values[:, n // group]
                    elif kind == "capped":
                        o = oracle.softmax_weights(oracle.cap(score[0], 2.0), seen) @ values[:, n // group]
                    else:
                        one, two = (oracle.softmax_weights(x, seen) @ values[:, n // group] for x in score)
                        o = torch.zeros_like(one)
                        o[:, :vdim] = oracle.rms((one - 0.7 * two)[:, :vdim], 1e-3) * 0.4
                        o *= torch.sigmoid(gate[lo:hi, n].double().cpu())[:, None]
                    want[lo:hi, n] = o
            for splits in (0, 1, 2, 5):
                out = torch.full((batch.tokens, heads * dv + 5), 7.0, device="cuda", dtype=dt)
                rows = (cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run,
                        min(batch.max_end, chunk) if chunk else batch.max_end, kv_heads, dv, chunk, scale)
                if kind == "paired":
                    hip.paired_attention(q, *rows, 0.7, 0.4, 1e-3, vdim, gate, out, splits)
                elif kind == "capped":
                    hip.capped_attention(q[:, :, 0].contiguous(), *rows, 2.0, out, splits)
                else:
                    hip.sigmoid_attention(q[:, :, 0].contiguous(), *rows, bias, out, splits)
                assert (out[:, heads * dv :] == 7.0).all()
                got = out[:, : heads * dv].view(-1, heads, dv)
                assert max_error(got, want) < (2e-5 if dtype == "float32" else 3e-2), (starts, lens, chunk, splits)


@pytest.mark.gpu
@pytest.mark.parametrize("y_dtype,dtype", [("float32", "float32"), ("float32", "bfloat16"), ("bfloat16", "bfloat16")])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,taps,rot,ff", [
    (1, 1, 1, 1, 0, 0, 0), (4, 2, 12, 20, 3, 8, 30), (6, 3, 48, 16, 4, 48, 256), (33, 1, 80, 40, 2, 12, 1000),
    (5, 5, 32, 130, 7, 16, 20003), (64, 8, 128, 128, 4, 64, 2064), (2, 2, 16, 8, 1, 6, 8),
])
def test_prepared_rows_at_any_position(heads, kv_heads, dim, vdim, taps, rot, ff, y_dtype, dtype):
    """Steps of several sequences, their first from position 0, beyond a million and in between:
    bias, convolution, norm, rotation and cache rows; PolyNorm beside them."""
    from petals_amd.ops import scores

    torch.manual_seed(0)
    hip, dt, ydt, eps, factor = scores.hip(), getattr(torch, dtype), getattr(torch, y_dtype), 1e-4, 1.3
    dk, dv = -(-dim // 32) * 32, -(-vdim // 16) * 16
    nq, nk, nv = heads * dk, kv_heads * dk, kv_heads * dv
    columns, at_up, ffp = nq + nk + nv, nq + nk + nv + 8, -(-ff // 8) * 8
    rot_config = {"base": 3000.0, "dims": rot}
    quarters = torch.tensor([f * 2 / math.pi for f in oracle.frequencies(rot_config)[0]], dtype=F64).cuda()
    live = torch.zeros(columns, dtype=torch.bool)
    for at, n, size, padded in ((0, heads, dim, dk), (nq, kv_heads, dim, dk), (nq + nk, kv_heads, vdim, dv)):
        live[at : at + n * padded].view(n, padded)[:, :size] = True
    bias = torch.randn(columns) * live if taps != 1 else None
    norm = torch.randn(nq + nk) * live[: nq + nk] if taps != 2 else None
    conv_w = torch.randn(taps, columns) * live if taps else None
    state = torch.full((6, taps, columns), 9.0, device="cuda") if taps > 1 else None
    cache = torch.full((15, PAGE_SIZE, nk + nv), 7.0, device="cuda", dtype=dt)
    act = [0.7, -0.4, 1.2, 0.3]
    # sequence: first position, sizes of its steps, pages, slot
    plan = [(0, [70, 1, 30, 1], [3, 5], 4), (1_000_000, [1, 9, 1, 1], [0] * 15625 + [8], 0),
            (61, [2, 1, 600, 1], [1, 2, 4, 6, 7, 9, 10, 11, 0, 12, 13], 2)]
    ys = [torch.randn(sum(steps), -(-(at_up + ff) // 8) * 8) for _, steps, _, _ in plan]
    for y in ys:
        y[:, :columns] *= live
        y[:, at_up + ff :] = 0
    ys = [y.to(ydt) for y in ys]
    want = []
    for y, (start, steps, _, _) in zip(ys, plan):
        u = y[:, :columns].double() + (0 if bias is None else bias.double())
        x = u if not taps else oracle.short_conv(u, conv_w.double().T.contiguous())
        pos = torch.arange(len(y)) + start
        q, k, v = x.split([nq, nk, nv], dim=1)
        if norm is not None:
            size = (heads * dim, kv_heads * dim)
            q, k = (t / torch.sqrt(t.pow(2).sum(-1, keepdim=True) / n + eps) * w for t, n, w in
                    zip((q, k), size, norm.double().split([nq, nk])))
        parts = [oracle.rotate(t.reshape(len(y), -1, dk), pos, rot_config) for t in (q, k)]
        for t in parts:
            t[:, :, :rot] *= factor
        want.append((parts[0].flatten(1), torch.cat([parts[1].flatten(1), v], dim=1)))
    # what the convolution takes from before a first position that is not 0: nothing was there, so zeros in the slot
    if state is not None:
        state[0] = 0
        state[2] = 0
    at = [0] * 3
    dev = [None if t is None else t.cuda() for t in (bias, conv_w, norm)]
    tol = 2e-5 if dtype == "float32" else 1e-2
    for step in range(4):
        who = [0, 1, 2] if step != 1 else [2, 0, 1]
        lens = [plan[i][1][step] for i in who]
        batch = PagedBatch([plan[i][2] for i in who], [plan[i][0] + at[i] for i in who], lens, torch.device("cuda"),
                           [plan[i][3] for i in who])
        y = torch.cat([ys[i][at[i] : at[i] + n] for i, n in zip(who, lens)]).cuda()
        single = batch.decode_only
        out = torch.full((len(y), ffp + 16), 5.0, device="cuda", dtype=ydt)
        view = out[:, 8 : 8 + ffp]
        q = hip.prepare_rows(
            y, cache, batch.pos, batch.owner, batch.tables, heads, kv_heads, dk, dim, nv, *dev, quarters, factor, state,
            batch.slot if state is not None else None, single, None if single else batch.tiles(16),
            None if single else batch.chunk_bounds(16), act if ff else [], at_up, ff, view if ff else None, eps,
        )
        for (lo, hi), i, n in zip(batch.row_ranges(), who, lens):
            rows = slice(at[i], at[i] + n)
            assert max_error(q[lo:hi], want[i][0][rows]) < tol
            pos = torch.arange(plan[i][0] + at[i], plan[i][0] + at[i] + n)
            got = cache[torch.tensor(plan[i][2])[pos // PAGE_SIZE], pos % PAGE_SIZE]
            assert max_error(got, want[i][1][rows]) < tol
            if ff:
                z = ys[i][rows, at_up : at_up + ff].double()
                a = oracle.poly_norm(z, torch.tensor(act, dtype=F64), eps)
                assert max_error(view[lo:hi, :ff], a) < (1e-5 if ydt == torch.float32 else 1e-2)
                assert (out[:, :8] == 5.0).all() and (out[:, 8 + ffp :] == 5.0).all()
            at[i] += n
    if state is not None:
        assert (state[[1, 3, 5]] == 9.0).all()


@pytest.mark.gpu
@pytest.mark.parametrize("t,d,groups", [(1, 8, 2), (5, 1000, 8), (600, 264, 3), (3, 4096, 2), (2, 131, 131), (700, 4096, 16), (4, 90, 6)])
def test_norm_in_groups_kernel(t, d, groups):
    from petals_amd.ops import scores

    torch.manual_seed(0)
    x0, y = torch.randn(t, d, device="cuda") * torch.linspace(0.1, 3, d, device="cuda"), torch.randn(t, d, device="cuda")
    w = torch.randn(d, device="cuda")
    for f32 in (True, False):
        x = x0.clone()
        h = scores.hip().residual_norm(x, y, None, w, d, 1e-3, f32, 1.0, groups)
        want = x0.double() + y.double()
        assert (x.double() - want).abs().max() < 1e-5
        want = oracle.group_norm(want, w.double(), groups, 1e-3)
        assert h.shape[1] % 8 == 0 and (h[:, d:] == 0).all()
        assert (h[:, :d].double() - want).abs().max() < (1e-4 if f32 else 1e-2) * want.abs().max()


@pytest.mark.gpu
def test_kernels_refuse_shapes_that_do_not_fit():
    from petals_amd.ops import scores

    hip = scores.hip()
    batch = PagedBatch([[0]], [0], [4], torch.device("cuda"))
    cache = torch.zeros(2, PAGE_SIZE, 48, device="cuda", dtype=torch.bfloat16)
    q = torch.zeros(4, 2, 32, device="cuda", dtype=torch.bfloat16)
    rows = (batch.pos, batch.owner, batch.tables, batch.tiles(4), 4, 4, 1, 16, 0, 1.0)
    with pytest.raises(RuntimeError):  # a narrow result
        hip.capped_attention(q, cache, *rows, 1.0, torch.zeros(4, 31, device="cuda"))
    with pytest.raises(RuntimeError):  # a cache of another width
        hip.sigmoid_attention(q, cache[..., :40].contiguous(), *rows, torch.zeros(2, device="cuda"), torch.zeros(4, 32, device="cuda"))
    with pytest.raises(RuntimeError):  # a bias for other heads
        hip.sigmoid_attention(q, cache, *rows, torch.zeros(3, device="cuda"), torch.zeros(4, 32, device="cuda"))
    with pytest.raises(RuntimeError):  # one map
        hip.paired_attention(q, cache, *rows, 0.5, 0.5, 1e-5, 16, None, torch.zeros(4, 32, device="cuda"))


@pytest.mark.gpu
def test_decode_graph_replays_match_eager(tmp_path, monkeypatch):
    """Replays with other work between them, requests coming and going; capturing
    a graph leaves every sequence's state as it was."""
    m = Model(tmp_path, SHAPES["mixed"], ("cuda", "bfloat16"))
    ids = [ids_of(90, seed=i) for i in range(3)]
    outs = {}
    for graphs in (True, False):
        if not graphs:
            monkeypatch.setenv("PETALS_AMD_NO_GRAPHS", "1")
        seqs = [m.engine.pool.open() for _ in ids]
        outs[graphs] = []
        for i in range(90):
            now = [0, 1, 2] if i % 7 else [0, 1]
            ys = m.engine.step(
                m.uids, [StepEntry(seqs[k], m.embed([ids[k][seqs[k].length]]), seqs[k].length) for k in now]
            )
            torch.randn(1000, device="cuda").sum().item()
            outs[graphs] += ys
        for s in seqs:
            s.close()
    assert len(m.engine._graphs) == 2
    for a, b in zip(outs[True], outs[False]):
        m.check(m.residual(a), m.residual(b), slack=0.5)
