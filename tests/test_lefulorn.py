"""Lefulorn against its plain oracle (tests/lefulorn_oracle.py): mechanisms alone,
and whole models through the span engine that serves them - prompts, portions,
decoding, mixed batches, pages and state slots used again - on the CPU path and,
marked gpu, on the HIP kernels in float32 and bfloat16."""

import math
import random

import pytest
import torch

import lefulorn_oracle as oracle
from petals_amd.models.config_base import load_model_config
from petals_amd.ops import reference
from petals_amd.server.from_pretrained import load_pretrained_block
from petals_amd.server.memory_cache import AllocationFailed
from petals_amd.server.paged_cache import PAGE_SIZE, PagedBatch, PagedPool
from petals_amd.server.span_engine import SpanEngine, StepEntry

PATHS = [
    ("cpu", "float32"),
    pytest.param(("cuda", "float32"), marks=pytest.mark.gpu),
    pytest.param(("cuda", "bfloat16"), marks=pytest.mark.gpu),
]
TOLERANCE = {"float32": 2e-4, "bfloat16": 5e-2}  # of the residual's own size

D, A = oracle.delta_layer, oracle.attention_layer
SHAPES = {
    # grouped heads, three mixing layers and one that does not mix, every kind of layer with and without an MLP
    "mixed": [
        D(heads=4, kv_heads=2, dim=12, vdim=20, conv=4),
        A(heads=6, kv_heads=2, dim=16, vdim=12, window=20),
        D(heads=3, kv_heads=3, dim=24, vdim=8, conv=2, ff=24),
        A(heads=4, kv_heads=4, dim=40, vdim=16, window=33, v_mix=False, every=50, coef=0.9),
        A(heads=4, kv_heads=2, dim=8, vdim=12, window=9, ff=None, scale=0.5),
        D(heads=6, kv_heads=1, dim=16, vdim=16, conv=3),
        A(heads=2, kv_heads=2, dim=16, vdim=12, window=70, coef=0.1, every=3),
    ],
    # everything that can be one is one
    "ones": [
        D(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, ff=1),
        A(heads=1, kv_heads=1, dim=1, vdim=1, window=1, every=1, ff=1),
        D(heads=1, kv_heads=1, dim=1, vdim=1, conv=2),
    ],
    # equal sizes everywhere
    "equal": [D(heads=32, kv_heads=32, dim=32, vdim=32, conv=4, ff=32)]
    + [A(heads=32, kv_heads=32, dim=32, vdim=32, window=32, every=32, ff=32)] * 2,
    # more heads on one key than a tile has rows, head sizes that are no multiple of anything
    "wide": [
        D(heads=10, kv_heads=5, dim=70, vdim=133, conv=5),
        A(heads=72, kv_heads=1, dim=33, vdim=65, window=100),
        A(heads=20, kv_heads=1, dim=72, vdim=65, window=50),
    ],
    # heads beyond the tiled kernels' sizes
    "long_heads": [
        A(heads=2, kv_heads=1, dim=270, vdim=24, window=50, scale=0.05),
        D(heads=2, kv_heads=1, dim=270, vdim=270, conv=4),
        D(heads=1, kv_heads=1, dim=24, vdim=2100, conv=2),
        A(heads=2, kv_heads=2, dim=24, vdim=260, window=50, v_mix=False),
    ],
    "no_attention": [D(ff=30), D(heads=2, kv_heads=2, conv=1)],
    "no_recurrence": [A(), A(heads=3, kv_heads=3, window=7), A(heads=6, kv_heads=6, v_mix=False)],
}
SHAPES["no_recurrence"][1]["mixer"].update(kv_heads=3, vdim=8)  # 3 x 8 against 2 x 12: equal only as a product


class Model:
    """A random model served by a SpanEngine, and its oracle."""

    def __init__(self, tmp_path, layers, path=("cpu", "float32"), *, width=40, vocab=97, tokens=1024, seed=0, edit=None,
                 eps=1e-6, sequences=None, ranks=(6, 5)):
        self.device, self.dtype = path
        self.raw = oracle.config_dict(vocab=vocab, width=width, layers=layers, eps=eps)
        self.weights = oracle.random_model(self.raw, seed, *ranks)
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
        x = self.weights["embed"][torch.as_tensor(ids)].float().to(self.device)
        return torch.nn.functional.pad(x, (0, self.config.stream_width - x.shape[1]), value=7.0)  # the rest is not read

    def residual(self, y):
        return y[..., : self.config.hidden_size].detach().double().cpu()

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


@pytest.mark.parametrize("taps", [1, 2, 4])
def test_short_conv(taps):
    x, w = torch.randn(2, 9, 5).double(), torch.randn(5, taps).double()
    padded = torch.cat([torch.zeros(2, taps - 1, 5).double(), x], dim=1)
    got = reference.short_conv(padded, w)
    for b in range(2):
        assert torch.allclose(got[b], oracle.short_conv(x[b], w))
    # a later portion, with the inputs before it ahead
    assert torch.allclose(reference.short_conv(padded[:, 4:], w), got[:, 4:])


def test_gated_delta_rule_and_its_state():
    s, h, dim, vdim = 11, 2, 6, 4
    q, k, g = (torch.randn(s, h, dim).double() for _ in range(3))
    v, beta, g = torch.randn(s, h, vdim).double(), torch.rand(s, h).double(), torch.sigmoid(g)
    want = oracle.delta_rule(q, k, v, g, beta)
    args = [t[None].float() for t in (q, k, v, g, beta)]
    got, _ = reference.gated_delta_rule(*args)
    assert torch.allclose(got[0].double(), want, atol=1e-4)
    first, state = reference.gated_delta_rule(*(t[:, :4] for t in args))
    rest, _ = reference.gated_delta_rule(*(t[:, 4:] for t in args), state)
    assert torch.allclose(torch.cat([first, rest], 1), got, atol=1e-5)


def test_decay_is_one_per_channel():
    h, a1, a2 = torch.randn(3, 8).double(), torch.randn(2, 8).double(), torch.randn(6, 2).double()
    g = oracle.channel_decay(h, a1, a2, torch.tensor([0.3, -0.2]).double(), torch.randn(6).double(), 2, 3)
    assert g.shape == (3, 2, 3) and (g > 0).all() and (g < 1).all() and len(g.unique()) == 18


def test_unit_vectors():
    x = torch.randn(3, 2, 7)
    x[0] = 0
    assert torch.allclose(reference.unit_vectors(x).double(), oracle.unit(x.double()), atol=1e-6)


def test_query_temperature_steps_at_multiples():
    pos = torch.arange(60)
    for coef, every in ((0.5, 16), (0.3, 1), (0.0, 7)):
        got = reference.query_temperature(pos, coef, every)
        assert torch.allclose(got.double(), oracle.temperature(pos.double(), coef, float(every)), atol=1e-6)
    got = reference.query_temperature(pos, 0.5, 16)
    assert got[14] == 1 and got[15] > 1 and got[15] == got[30] and got[31] > got[30]


@pytest.mark.parametrize("heads", [1, 3, 8, 12])
def test_slopes(heads):
    got = reference.distance_slopes(heads)
    assert torch.allclose(got.double(), torch.tensor([oracle.slope(h, heads) for h in range(heads)]).double())


@pytest.mark.parametrize("window,start", [(1, 0), (4, 0), (50, 0), (5, 9)])
def test_attention_with_bias_and_sink(window, start):
    """A portion's queries against all keys, as the oracle's rows of a whole sequence."""
    s, heads, kv, dim, vdim = 20, 4, 2, 6, 3
    q, k, v = (torch.randn(s, n, m).double() for n, m in ((heads, dim), (kv, dim), (kv, vdim)))
    sink = torch.randn(heads).double()
    pos = torch.arange(s)
    temp = oracle.temperature(pos.double(), 0.4, 5.0)
    want = torch.zeros(s, heads, vdim).double()
    seen = oracle.window_mask(s, window)
    for n in range(heads):
        score = ((q[:, n] * temp[:, None]) @ k[:, n // 2].T) * 0.3
        score = score - oracle.slope(n, heads) * (pos[:, None] - pos[None, :])
        want[:, n] = oracle.sink_softmax(score.masked_fill(~seen, -math.inf), sink[n]) @ v[:, n // 2]
    got = reference.biased_sink_attention(
        q[start:].float(), k.float(), v.float(), pos[start:], pos, scale=0.3, window=window, sink=sink.float(),
        slopes=reference.distance_slopes(heads), temperature=reference.query_temperature(pos[start:], 0.4, 5),
    )
    assert torch.allclose(got.double(), want[start:], atol=1e-5)


def test_sink_takes_its_share_even_of_a_single_key():
    score, sink = torch.tensor([[2.0]]).double(), torch.tensor(2.0).double()
    assert torch.allclose(oracle.sink_softmax(score, sink), torch.tensor([[0.5]]).double())


# ------------------------------------------------------- configuration, loading


def test_config_reads_every_layer_and_rejects_nonsense(tmp_path):
    raw = oracle.config_dict(layers=SHAPES["mixed"], eps=0.25, logit_scale=0.3)
    oracle.save_model(str(tmp_path), raw, oracle.random_model(raw))
    cfg = load_model_config(str(tmp_path))
    assert cfg.model_type == "lefulorn" and cfg.hidden_size == 40 and cfg.layer_norm_eps == 0.25
    assert cfg.logit_scale == 0.3 and cfg.num_blocks == 7 and not cfg.rewindable
    assert [cfg.spec(i).mixer.taps for i in (0, 2, 5)] == [4, 2, 3]
    assert [cfg.spec(i).mixer.window for i in (1, 3, 4, 6)] == [20, 33, 9, 70]
    assert cfg.spec(3).mixer.temp_every == 50 and cfg.spec(0).mlp is None and cfg.spec(2).mlp.ff == 24
    assert cfg.first_mixing_layer == 1 and cfg.stream_width == 40 + 24
    assert cfg.cache_values_per_token(0) == 0 and cfg.cache_values_per_token(3) == 4 * (64 + 16)
    assert cfg.state_shapes(0) == {"delta": (4, 16, 32), "conv": (4, 2 * 24 + 80)} and cfg.state_shapes(1) == {}
    assert cfg.valid_cuts() is None  # a chain may be cut anywhere
    again = type(cfg).from_hf_dict(cfg.to_dict())  # what a server announces
    assert again.spec(4) == cfg.spec(4) and again.stream_width == 64 and again.logit_scale == 0.3
    for bad in (
        [A(heads=3, kv_heads=2)], [D(dim=0)], [D(conv=0)], [A(window=-1)], [A(every=0)], [A(every=1.5)],
        [{**A(), "type": "convolution"}], [A(), A(vdim=16)],
        [{**A(), "mlp": {"kind": "moe", "ff": 4}}],
    ):
        with pytest.raises(ValueError):
            type(cfg).from_hf_dict(oracle.config_dict(layers=bad))
    alone = type(cfg).from_hf_dict(oracle.config_dict(layers=[A(), A(v_mix=False), A(v_mix=False)]))
    assert alone.stream_width == 40 and alone.rewindable  # nothing to mix with: nothing travels


def test_loader_refuses_incomplete_checkpoints(tmp_path):
    raw = oracle.config_dict(layers=[D(), A()])
    for i, name, shape in ((0, "l0.mix.k.conv", (24, 3)), (0, "l0.mix.a2", (48, 7)), (1, "l1.mix.sink", (5,))):
        weights = oracle.random_model(raw)
        keep = weights.pop(name)
        oracle.save_model(str(tmp_path), raw, weights)
        with pytest.raises(KeyError, match=name[3:]):
            load_pretrained_block(str(tmp_path), load_model_config(str(tmp_path)), i)
        assert keep.shape != shape
        weights[name] = torch.zeros(shape, dtype=keep.dtype)
        oracle.save_model(str(tmp_path), raw, weights)
        with pytest.raises(ValueError, match="config says"):
            load_pretrained_block(str(tmp_path), load_model_config(str(tmp_path)), i)


def test_random_weights_without_a_checkpoint():
    from petals_amd.models.lefulorn.config import LefulornConfig
    from petals_amd.server.from_pretrained import build_empty_block, init_random_block_

    cfg = LefulornConfig.from_hf_dict(oracle.config_dict(layers=SHAPES["mixed"]), name_or_path="random")
    for i in range(cfg.num_blocks):
        block = build_empty_block(cfg, i, torch.device("cpu"), torch.float32)
        init_random_block_(block, cfg, i)
        assert torch.isfinite(block(torch.randn(1, 9, cfg.stream_width))).all()


# ------------------------------------------------------------- whole models


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_prompt_matches_oracle(tmp_path, shape, path):
    m = Model(tmp_path, SHAPES[shape], path)
    ids = ids_of(110)
    want = m.expected(ids)
    m.check(m.run(ids), want)
    m.check(m.run(ids, [90] + [1] * 20), want)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("width,vocab,eps,ranks", [(8, 11, 1e-6, (1, 1)), (131, 40, 1e-3, (16, 9)), (256, 300, 0.3, (70, 8))])
def test_other_widths_eps_and_ranks(tmp_path, width, vocab, eps, ranks, path):
    m = Model(tmp_path, SHAPES["mixed"], path, width=width, vocab=vocab, eps=eps, seed=3, ranks=ranks)
    ids = ids_of(90, vocab)
    want = m.expected(ids)
    slack = 2.0 if width == 8 else 1.0  # a norm over a handful of values amplifies rounding
    m.check(m.run(ids), want, slack)
    m.check(m.run(ids, [70] + [1] * 20), want, slack)


@pytest.mark.parametrize("path", PATHS[:2])
def test_every_fault_would_show(tmp_path, path):
    """The inputs of these tests tell each planted mistake from the design."""
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = ids_of(110)
    got = m.run(ids)
    for fault in (
        "conv_reversed", "conv_one_less", "decay_after", "no_delta", "read_before_write", "head_interleave", "window+1",
        "window-1", "no_sink", "no_mix", "mix_with_last", "no_temp", "temp_edge", "no_bias", "key_bias", "no_gate",
        "no_square",
    ):
        assert m.error(got, m.expected(ids, [fault])) > 20 * TOLERANCE[m.dtype], fault


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("cuts", [
    [1] * 140, [100] + [1] * 40, [2] * 70, [2, 3, 64, 1, 63, 2, 5], [64, 64, 12], [63, 65, 12], [9, 131], [139, 1],
    [16] * 8 + [12], [17] * 8 + [4], [3, 1] * 35,
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


def standing_out(layer=0, query=90, key=91):
    """Weights under which token `query` scores far higher on token `key` than on
    any other, so that one key decides the attention of one row."""

    def edit(w):
        p = f"l{layer}.mix."
        w["embed"][:, :2] = 0
        w["embed"][query, 0] = 6.0
        w["embed"][key, 1] = 6.0
        w[f"l{layer}.norm1"][:2] = 1.0
        for name, dim in (("q", 0), ("k", 1)):
            w[p + name][:] = 0
            w[p + name][:, dim] = 2.0
            w[p + name + ".b"][:] = 0

    return edit


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("window", [2, 33, 64, 65, 130])
def test_keys_just_inside_and_just_outside_the_window(tmp_path, window, path):
    layer = A(heads=2, kv_heads=1, dim=16, window=window, ff=None, scale=0.25)
    m = Model(tmp_path, [layer], path, edit=standing_out())
    for place in (window, window + 1, 127 + window, 128 + window):  # the query's position: edges of pages and batches
        for gap in (window - 1, window):
            ids = ids_of(place + 3, vocab=80)
            ids[place], ids[place - gap] = 90, 91
            want = m.expected(ids)
            if gap > 0:
                wrong = m.expected(ids, ["window-1" if gap == window - 1 else "window+1"])
                assert m.error(want[place : place + 1], wrong[place : place + 1]) > 0.15
            for cuts in ([len(ids)], [place, 1, 2], [place - 1, 2, 2] if place > 1 else [1] * len(ids)):
                m.check(m.run(ids, cuts), want)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("heads", [1, 17])
def test_far_keys_and_page_borders(tmp_path, path, heads):
    """One key among hundreds, at and around the borders of pages and tiles."""
    m = Model(tmp_path, [A(heads=heads, kv_heads=1, dim=16, window=600, ff=None, scale=0.5)], path, edit=standing_out())
    n = 520
    for key in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 447, 448, 511)[:: 1 if heads == 1 else 3]:
        ids = ids_of(n, vocab=80)
        ids[key], ids[n - 1] = 91, 90
        want = m.expected(ids)
        assert m.error(want[-1:], m.expected(ids[:key] + [5] + ids[key + 1 :])[-1:]) > 0.15  # without that key
        for cuts in ([n], [n - 1, 1], [300, 219, 1]):
            m.check(m.run(ids, cuts), want)


def slow_decay(w):
    for name, t in w.items():
        if name.endswith("A_log"):
            t.fill_(-9.0)


@pytest.mark.parametrize("path", PATHS)
def test_state_remembers_the_first_token(tmp_path, path):
    """Decays close to one: the first token still shows hundreds of tokens later,
    however the tokens between are cut."""
    layer = D(heads=4, kv_heads=2, dim=32, vdim=16, conv=3)
    m = Model(tmp_path, [layer], path, edit=slow_decay)
    pair = [ids_of(260, vocab=3, seed=7), None]
    pair[1] = [96] + pair[0][1:]
    wants = [m.expected(ids) for ids in pair]
    late = m.errors(wants[0][-40:], wants[1][-40:])
    assert float(late.mean()) > 0.05
    for ids, want in zip(pair, wants):
        for cuts in ([260], [1] * 20 + [240], [100, 2, 3, 16, 129] + [1] * 10):
            m.check(m.run(ids, cuts), want, slack=0.3)


@pytest.mark.parametrize("path", PATHS)
def test_strong_decays_do_not_overflow(tmp_path, path):
    def edit(w):
        w["l0.mix.A_log"][:] = torch.tensor([5.0, -2.0, 3.0, 1.0])
        w["l0.mix.a2"] *= 4

    m = Model(tmp_path, [D(heads=4, kv_heads=2, dim=32, vdim=16, conv=3)], path, edit=edit)
    ids = ids_of(100)
    m.check(m.run(ids), m.expected(ids))
    m.check(m.run(ids, [37] + [1] * 10 + [53]), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_first_tokens(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    for n in (1, 2, 3, 4, 5):
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
    # without a recurrent layer the pages roll back as those of other families
    m = Model(tmp_path, SHAPES["no_recurrence"], path)
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
def test_chains_cut_anywhere(tmp_path, path):
    """The span in two engines, as two servers would run it: the mixed-in values travel in the stream."""
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = ids_of(60)
    for cut in (2, 4, 6):
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
    cached = m.engine.forward(m.uids, x)
    plain = x
    for uid in m.uids:
        plain = m.engine.blocks[uid](plain)
    for i, t in enumerate(ids):
        m.check(m.residual(cached[i]), m.expected(t))
        m.check(m.residual(plain[i]), m.expected(t))


# ------------------------------------------------------------- pool and batch


def test_pool_slots_and_bytes():
    pool = PagedPool(
        {1: 32}, 3, dtype=torch.float32, device="cpu", max_sequences=2, states={0: {"delta": (2, 16, 16), "conv": (3, 10)}}
    )
    assert pool.bytes_per_sequence == 4 * (512 + 30) and pool.total_bytes == 3 * 64 * 32 * 4 + 2 * 4 * 542
    a, b = pool.open(), pool.open()
    assert {a.slot, b.slot} == {0, 1} and pool.scratch_slot == 2 and not pool.can_open(1)
    assert pool.state(0)["delta"].shape == (3, 2, 16, 16)
    a.close()
    a.close()
    c = pool.open()
    assert c.slot == a.slot and pool.live_sequences == 2
    with pytest.raises(ValueError, match="not in this server's span"):
        pool.state(1)


def test_chunk_bounds():
    batch = PagedBatch([[0], [1], [2]], [0, 5, 9], [33, 1, 16], torch.device("cpu"), [4, 2, 0])
    batch._host_ints = lambda v: torch.tensor(v, dtype=torch.int32)
    assert batch.chunk_bounds(16).tolist() == [0, 3, 4, 5] and batch.slots == [4, 2, 0]
    assert batch.tiles(16).tolist() == [[0, 16], [16, 16], [32, 1], [33, 1], [34, 16]]


def test_sessions_wait_for_slots():
    import asyncio

    from petals_amd.server.memory_cache import MemoryCache
    from petals_amd.server.paged_cache import PageDescriptor

    async def main():
        pool = PagedPool({}, 4, dtype=torch.float32, device="cpu", max_sequences=2, states={0: {"delta": (1, 16, 16)}})
        cache = MemoryCache(10 * pool.total_bytes, torch.device("cpu"))
        async with cache.allocate_cache(PageDescriptor(pool, 1, 65)):
            with pytest.raises(AllocationFailed):
                async with cache.allocate_cache(PageDescriptor(pool, 2, 1), timeout=0.05):
                    pass
            async with cache.allocate_cache(PageDescriptor(pool, 1, 1), timeout=0.05):
                assert pool.live_sequences == 2
        async with cache.allocate_cache(PageDescriptor(pool, 2, 1), timeout=0.05):
            pass
        assert pool.live_sequences == 0 and cache.current_size_bytes == 0

    asyncio.new_event_loop().run_until_complete(main())


# --------------------------------------------------------- kernels, one by one


@pytest.mark.gpu
@pytest.mark.parametrize("heads,kv,dim,vdim,window,dtype", [
    (1, 1, 32, 16, 0, "bfloat16"), (8, 4, 64, 64, 45, "bfloat16"), (12, 12, 128, 128, 64, "bfloat16"),
    (40, 2, 96, 80, 100, "bfloat16"), (70, 1, 160, 48, 100, "bfloat16"), (6, 2, 256, 256, 33, "bfloat16"),
    (3, 1, 288, 32, 33, "bfloat16"), (6, 3, 64, 48, 50, "float32"),
])
def test_paged_attention_kernel(heads, kv, dim, vdim, window, dtype):
    """Every key split and both row layouts agree with the dense computation, on scattered pages."""
    from petals_amd.ops import hybrid

    torch.manual_seed(0)
    dt = getattr(torch, dtype)
    scale = 1.5 * dim**-0.5
    cache = torch.randn(9, PAGE_SIZE, kv * (dim + vdim), device="cuda").to(dt)
    slopes, sink = reference.distance_slopes(heads, "cuda"), torch.randn(heads, device="cuda")
    for starts, lens in (([0, 130, 63], [40, 1, 70]), ([0, 130, 63], [1, 1, 1])):
        pages = [[3], [5, 0, 7], [8, 1, 2]]
        batch = PagedBatch(pages, starts, lens, torch.device("cuda"))
        q = torch.randn(batch.tokens, heads, dim, device="cuda").to(dt)
        gate = torch.randn(batch.tokens, heads * vdim + 8, device="cuda").to(dt)[:, 8:]
        want = torch.empty(batch.tokens, heads, vdim, dtype=torch.float64)
        for (lo, hi), p, s in zip(batch.row_ranges(), pages, starts):
            rows = cache[p].reshape(-1, kv * (dim + vdim))[: s + hi - lo].double().cpu()
            k, v = rows[:, : kv * dim].view(-1, kv, dim), rows[:, kv * dim :].view(-1, kv, vdim)
            gap = (torch.arange(len(rows))[s:, None] - torch.arange(len(rows))[None, :]).double()
            seen = oracle.window_mask(len(rows), window or len(rows))[s:]
            for n in range(heads):
                g = n // (heads // kv)
                score = q[lo:hi, n].double().cpu() @ k[:, g].T * scale - oracle.slope(n, heads) * gap
                p_ = oracle.sink_softmax(score.masked_fill(~seen, -math.inf), sink[n].double().cpu())
                want[lo:hi, n] = p_ @ v[:, g]
        want = want.flatten(1) * torch.sigmoid(gate.double().cpu())
        run = batch.run_tokens(heads // kv)
        for splits in (0, 1, 2, 5):
            got = hybrid.hip().paged_attention(
                q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, batch.max_end, kv, vdim, window,
                scale, slopes, sink, gate, dtype == "float32", splits,
            )
            assert (got.double().cpu() - want).abs().max() < (2e-5 if dtype == "float32" else 3e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("heads,kv,dim,vdim,taps", [
    (1, 1, 1, 1, 1), (4, 2, 12, 20, 4), (10, 5, 64, 64, 3), (4, 1, 128, 128, 4), (2, 1, 200, 48, 2), (2, 2, 16, 300, 5),
])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_delta_kernels(heads, kv, dim, vdim, taps, dtype):
    """Chunks, then single tokens, from projections given as such; scattered slots."""
    from petals_amd.ops import hybrid

    torch.manual_seed(0)
    hip, dt = hybrid.hip(), getattr(torch, dtype)
    sizes = [kv * dim, kv * dim, heads * vdim, heads]
    gap = 8 if dim % 8 == 0 else 3  # aligned columns and others
    cols = [0, kv * dim + gap, 2 * kv * dim + gap, 2 * kv * dim + heads * vdim + gap]
    rank, g_rank = 8, 16
    at_a = -(-(cols[3] + heads) // 8) * 8
    at_g = at_a + rank
    width = at_g + g_rank
    lens = [37, 1, 16, 50]
    total, tail = [x + 5 for x in lens], 5
    ys = [torch.randn(n, width).to(dt) for n in total]
    conv_w = torch.randn(sum(sizes[:3]), taps)
    a2, g2 = torch.randn(heads * dim, rank).to(dt), torch.randn(heads * vdim, g_rank).to(dt)
    a_log, dt_bias, norm_w = torch.randn(heads) - 1, torch.randn(heads * dim) - 1, 1 + 0.3 * torch.randn(vdim)
    eps = 1e-5
    wants = []
    for y in ys:
        y = y.double()
        parts = [y[:, c : c + n] for c, n in zip(cols, sizes)]
        w = dict(zip("qkv", conv_w.double().split(sizes[:3])))
        q, k, v = (oracle.silu(oracle.short_conv(p, w[n])) for p, n in zip(parts, "qkv"))
        of = torch.arange(heads) // (heads // kv)
        q = oracle.unit(q.view(-1, kv, dim))[:, of] * dim**-0.5
        k = oracle.unit(k.view(-1, kv, dim))[:, of]
        eye = torch.eye(width).double()
        g = oracle.channel_decay(y, eye[at_a : at_a + rank], a2.double(), a_log.double(), dt_bias.double(), heads, dim)
        o = oracle.delta_rule(q, k, v.view(-1, heads, vdim), g, torch.sigmoid(parts[3]))
        gate = torch.sigmoid(y[:, at_g : at_g + g_rank] @ g2.double().T).view(-1, heads, vdim)
        wants.append((oracle.norm(o, norm_w.double(), eps) * gate).flatten(1))
    up = lambda n: -(-n // 16) * 16
    slots = [5, 0, 3, 1]
    delta = torch.full((7, heads, up(dim), up(vdim)), 9.0, device="cuda")  # what a slot's last user left
    for s in slots:  # padding stays zero in a pool's life
        delta[s, :, dim:] = 0
        delta[s, :, :, vdim:] = 0
    conv = torch.full((7, taps, conv_w.shape[0]), 9.0, device="cuda")
    cu = [t.cuda() for t in (conv_w.t().contiguous(), a_log.exp(), dt_bias, norm_w, a2, g2)]
    tol = 2e-4 if dtype == "float32" else 3e-2

    def batch_of(starts, counts):
        return PagedBatch([[0]] * 4, starts, counts, torch.device("cuda"), slots)

    def rel(got, want):
        return float((got.double().cpu() - want).abs().max() / want.abs().max())

    starts = [0] * 4
    for counts in ([20, 1, 2, 50], [17, 0, 14, 0]):
        live = [i for i in range(4) if counts[i]]
        b = PagedBatch([[0]] * len(live), [starts[i] for i in live], [counts[i] for i in live], torch.device("cuda"),
                       [slots[i] for i in live])
        y = torch.cat([ys[i][starts[i] : starts[i] + counts[i]] for i in live]).cuda()
        a = (y[:, at_a : at_a + rank].float() @ cu[4].float().T).contiguous()
        gate = (y[:, at_g : at_g + g_rank].float() @ cu[5].float().T).contiguous()
        o = hip.delta_prefill(y, a, cu[0], cu[1], cu[2], b.tiles(16), b.chunk_bounds(16), b.pos, b.owner, b.slot, delta,
                              conv, heads, kv, dim, vdim, cols)
        out = hip.delta_norm(o, gate, cu[3], heads, heads * vdim + 8, True, eps)
        assert (out[:, heads * vdim :] == 0).all()
        for i, (lo, hi) in zip(live, b.row_ranges()):
            assert rel(out[lo:hi, : heads * vdim], wants[i][starts[i] : starts[i] + hi - lo]) < tol
            starts[i] += hi - lo
    if not hip.delta_decodes(dim, vdim):
        return
    for step in range(tail):
        b = batch_of(starts, [1] * 4)
        y = torch.stack([t[s] for t, s in zip(ys, starts)]).cuda()
        out = hip.delta_decode(y, cu[0], cu[4], cu[5], at_a, at_g, cu[1], cu[2], cu[3], b.pos, b.slot, delta, conv,
                               heads, kv, dim, vdim, cols, heads * vdim, eps)
        for i in range(4):
            assert rel(out[i], wants[i][starts[i]]) < tol
            starts[i] += 1


@pytest.mark.gpu
@pytest.mark.parametrize("t,d,extra", [(1, 7, 0), (5, 128, 9), (600, 1000, 24), (3, 4097, 1)])
def test_residual_kernels(t, d, extra):
    from petals_amd.ops import hybrid

    torch.manual_seed(0)
    hip = hybrid.hip()
    x0, w, bias = torch.randn(t, d + extra, device="cuda"), torch.randn(d, device="cuda"), torch.randn(d, device="cuda")
    dp = -(-d // 8) * 8
    for y in (None, torch.randn(t, d + 5, device="cuda"), torch.randn(t, d + 5, device="cuda").bfloat16()):
        for b in (None, bias):
            x = x0.clone()
            h = hip.residual_norm(x, y, b, w, d, 1e-3, True)
            want = x0[:, :d].double()
            if y is not None:
                want = want + y[:, :d].double() + (0 if b is None else b.double())
            assert (x[:, :d].double() - want).abs().max() < 1e-5 and torch.equal(x[:, d:], x0[:, d:])
            assert (h[:, :d].double() - oracle.norm(want, w.double(), 1e-3)).abs().max() < 1e-4
            assert h.shape == (t, dp) and (h[:, d:] == 0).all()
    if t <= 8:
        parts, x = torch.randn(37, t, dp, device="cuda"), x0.clone()
        hip.residual_sum(parts, bias, x, d)
        want = x0[:, :d].double() + parts.double().sum(0)[:, :d] + bias.double()
        assert (x[:, :d].double() - want).abs().max() < 1e-4 and torch.equal(x[:, d:], x0[:, d:])
    y, b = torch.randn(t, dp, device="cuda"), torch.randn(dp, device="cuda")
    want = (y.double() + b.double()).clamp(min=0) ** 2
    assert (hip.bias_relu2(y.clone(), b).double() - want).abs().max() < 1e-4


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
