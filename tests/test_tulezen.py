"""Tulezen against its plain oracle (tests/tulezen_oracle.py): mechanisms alone,
and whole models through the span engine that serves them - prompts, portions,
decoding, mixed batches, pages used again - on the CPU path and, marked gpu, on
the HIP kernels in float32 and bfloat16."""

import random

import pytest
import torch

import tulezen_oracle as oracle
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

L = oracle.layer_dict
SHAPES = {
    # sharing across layers of different windows, a layer without experts, odd sizes
    "mixed": [
        L(heads=3, dim=16, vdim=24, kv_rank=40, window=20),
        L(heads=5, dim=8, vdim=8, kv_rank=56, window=70, experts=9, top=3, ff=24),
        L(heads=2, dim=24, vdim=16, kv_rank=40, window=33, kv_from=0, mlp=False),
        L(heads=4, dim=16, vdim=40, kv_rank=56, window=9, kv_from=1, limit=0.4),
    ],
    # everything that can be one is one
    "ones": [L(heads=1, dim=8, vdim=8, kv_rank=8, window=1, experts=1, top=1, ff=8),
             L(heads=1, dim=1, vdim=1, kv_rank=1, window=3, experts=2, top=2, ff=1)],
    # equal sizes everywhere, all experts taken, many heads
    "equal": [L(heads=32, dim=32, vdim=32, kv_rank=32, window=32, experts=4, top=4, ff=32),
              L(heads=32, dim=32, vdim=32, kv_rank=32, window=32, kv_from=0, experts=4, top=1, ff=32)],
    # more heads than one tile of rows, larger latent
    "wide": [L(heads=72, dim=8, vdim=16, kv_rank=200, window=100, experts=16, top=4, ff=56)],
    # latent beyond the tiled kernel's sizes
    "long_latent": [L(heads=2, dim=16, vdim=16, kv_rank=530, window=50)],
}


class Model:
    """A random model served by a SpanEngine, and its oracle."""

    def __init__(self, tmp_path, layers, path=("cpu", "float32"), *, width=40, vocab=97, tokens=1024, seed=0, edit=None,
                 eps=1e-6):
        self.device, self.dtype = path
        self.raw = oracle.config_dict(vocab=vocab, width=width, layers=layers, eps=eps)
        self.weights = oracle.random_model(self.raw, seed, decided=self.dtype == "bfloat16")
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
        pool = SpanEngine.pool_for(list(blocks.values()), tokens, dtype=dtype, device=self.device)
        self.engine = SpanEngine(blocks, pool, max_length=tokens)
        self.uids = tuple(blocks)

    def embed(self, ids):
        return self.weights["embed"][torch.as_tensor(ids)].float().to(self.device)

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
        return torch.cat(out).double().cpu()

    def errors(self, got, want):
        """RMS difference at each position, relative to the residual's RMS."""
        return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()

    def error(self, got, want):
        return float(self.errors(got, want).max())

    def check(self, got, want, slack=1.0):
        """All but a few positions within the tolerance, and none far from it:
        where a sublayer's output nearly cancels, the norm behind it amplifies
        16-bit rounding."""
        e, limit = self.errors(got, want), slack * TOLERANCE[self.dtype]
        assert float(e.max()) < 2.5 * limit and int((e > limit).sum()) <= 0.02 * len(e) + 1, e.topk(min(5, len(e)))


def ids_of(n, vocab=97, seed=1):
    return random.Random(seed).choices(range(vocab), k=n)


# ------------------------------------------------------------- mechanisms


def test_zero_centered_norm():
    x, w = torch.randn(5, 24), torch.randn(24) * 0.3
    for eps in (1e-6, 0.5):
        got = reference.zero_centered_rms_norm(x, w, eps).double()
        want = oracle.zero_centered_norm(x.double(), w.double(), eps)
        assert torch.allclose(got, want, atol=1e-5)
    assert not torch.allclose(got, oracle.zero_centered_norm(x.double(), w.double(), 0.5, {"plain_norm"}), atol=1e-2)


def test_clamped_swiglu_saturates_on_the_right_sides():
    g, u = torch.tensor([-9.0, -1.0, 0.5, 9.0]), torch.tensor([9.0, -9.0, 0.3, -0.2])
    got = reference.clamped_swiglu(g, u, 1.5)
    gc, uc = torch.tensor([-9.0, -1.0, 0.5, 1.5]), torch.tensor([1.5, -1.5, 0.3, -0.2])  # the gate has no floor
    assert torch.allclose(got, gc * torch.sigmoid(1.702 * gc) * (uc + 1))


def test_router_scores_are_softmax_over_all_experts():
    x, w = torch.randn(7, 16), torch.randn(6, 16)
    scores, chosen = reference.softmax_topk(x, w, 2)
    want_w, want_e = oracle.route(x.double(), w.double(), 2)
    assert torch.equal(chosen, want_e) and torch.allclose(scores.double(), want_w, atol=1e-6)
    assert (scores.sum(-1) < 1).all()


@pytest.mark.parametrize("window", [1, 2, 7, 50, 0])
def test_window_mask(window):
    full = reference.sliding_window_mask(40, 40, 0, window)
    assert torch.equal(full, oracle.window_mask(40, window or 40))
    part = reference.sliding_window_mask(5, 40, 35, window)  # a portion: queries at 35..39
    assert torch.equal(part, full[35:])


def test_config_reads_every_layer_and_rejects_nonsense(tmp_path):
    raw = oracle.config_dict(layers=SHAPES["mixed"], eps=0.25)
    oracle.save_model(str(tmp_path), raw, oracle.random_model(raw))
    cfg = load_model_config(str(tmp_path))
    assert cfg.model_type == "tulezen" and cfg.hidden_size == 40 and cfg.layer_norm_eps == 0.25
    assert [cfg.spec(i).attention.window for i in range(4)] == [20, 70, 33, 9]
    assert cfg.spec(2).moe is None and cfg.spec(1).moe.top == 3 and cfg.spec(3).moe.limit == 0.4
    assert cfg.valid_cuts() == {0, 4}
    assert [cfg.cache_values_per_token(i) for i in range(4)] == [64, 64, 0, 0]
    again = type(cfg).from_hf_dict(cfg.to_dict())  # what a server announces
    assert again.spec(3) == cfg.spec(3) and again.hidden_size == 40 and again.layer_norm_eps == 0.25
    for bad in (
        [L(kv_rank=32), L(kv_rank=40, kv_from=0)], [L(kv_from=0)], [L(), L(kv_from=0), L(kv_from=1)],
        [{**L(), "type": "convolution"}], [L(experts=2, top=3)],
    ):
        with pytest.raises(ValueError):
            type(cfg).from_hf_dict(oracle.config_dict(layers=bad))


def test_loader_refuses_incomplete_checkpoints(tmp_path):
    raw = oracle.config_dict(layers=[L()])
    weights = oracle.random_model(raw)
    del weights["l0.mlp.e3.up"]
    oracle.save_model(str(tmp_path), raw, weights)
    with pytest.raises(KeyError, match="e3.up"):
        load_pretrained_block(str(tmp_path), load_model_config(str(tmp_path)), 0)


# ------------------------------------------------------------- whole models


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_prompt_matches_oracle(tmp_path, shape, path):
    m = Model(tmp_path, SHAPES[shape], path)
    ids = ids_of(150)
    m.check(m.run(ids), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("width,vocab,eps", [(8, 11, 1e-6), (131, 40, 1e-3), (256, 300, 0.3)])
def test_other_widths_and_eps(tmp_path, width, vocab, eps, path):
    m = Model(tmp_path, SHAPES["mixed"], path, width=width, vocab=vocab, eps=eps, seed=3)
    ids = ids_of(90, vocab)
    slack = 2.0 if width == 8 else 1.0  # a norm over a handful of values amplifies rounding
    m.check(m.run(ids), m.expected(ids), slack)
    m.check(m.run(ids, [70] + [1] * 20), m.expected(ids), slack)


@pytest.mark.parametrize("path", PATHS[:2])
def test_every_fault_would_show(tmp_path, path):
    """The inputs of these tests tell each planted mistake from the design.
    (The large eps keeps a common factor of the experts' sum from cancelling in
    the norm behind it.)"""
    m = Model(tmp_path, SHAPES["mixed"], path, eps=0.5)
    ids = ids_of(150)
    got = m.run(ids)
    for fault in ("window+1", "window-1", "no_share", "renorm_router", "no_plus_one", "no_limit", "plain_norm"):
        if fault == "no_share":  # layers 2 and 3 have no latent of their own: use the other owner's
            raw = dict(m.raw, layers=[dict(e, mixer=dict(e["mixer"])) for e in m.raw["layers"]])
            for e in raw["layers"]:
                e["mixer"].pop("kv_from", None)
            weights = dict(m.weights)
            for i, src in ((2, 0), (3, 1)):
                weights[f"l{i}.mix.dkv"] = weights[f"l{src}.mix.dkv"]
                weights[f"l{i}.mix.dkv.norm"] = weights[f"l{src}.mix.dkv.norm"]
            res = []
            oracle.run(raw, weights, ids, residuals=res)
            wrong = res[-1]
        else:
            wrong = m.expected(ids, [fault])
        assert m.error(got, wrong) > 4 * TOLERANCE[m.dtype], fault


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("cuts", [
    [1] * 140, [100] + [1] * 40, [2] * 70, [2, 3, 64, 1, 63, 2, 5], [64, 64, 12], [63, 65, 12], [9, 131], [139, 1],
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
    m = Model(tmp_path, SHAPES["mixed"], path)
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
            seqs.setdefault(k, m.engine.pool.open())
            entries.append(StepEntry(seqs[k], m.embed(ids[k][at[k] : at[k] + n]), at[k]))
            at[k] += n
        for k, y in zip(now, m.engine.step(m.uids, entries)):
            outs[k].append(y)
            if not left[k]:
                seqs[k].close()
    for k in plans:
        m.check(torch.cat(outs[k]).double().cpu(), m.expected(ids[k]))
    assert m.engine.pool.free_pages == m.engine.pool.num_pages


@pytest.mark.parametrize("path", PATHS)
def test_pages_are_used_again_in_any_order(tmp_path, path):
    """A pool of five pages, scrambled and full of other requests' state."""
    m = Model(tmp_path, SHAPES["mixed"], path, tokens=5 * PAGE_SIZE)
    pool = m.engine.pool
    for round_, n in enumerate((320, 200, 129, 64, 65)):
        m.run(ids_of(n, seed=round_ + 50))
        random.Random(round_).shuffle(pool._free)
        ids = ids_of(200, seed=round_)
        m.check(m.run(ids, [100, 27, 1, 1, 71]), m.expected(ids))
    a, b = pool.open(), pool.open()
    m.run(ids_of(190), sequence=a)
    with pytest.raises(AssertionError, match="pages needed"):
        m.run(ids_of(190), sequence=b)
    a.close()
    ids = ids_of(190)
    m.check(m.run(ids, sequence=b), m.expected(ids))


def standing_out(window_layer=0, query=90, key=91):
    """Weights under which token `query` scores far higher on token `key` than
    on any other, so that one key decides the attention of one row."""

    def edit(w):
        p = f"l{window_layer}.mix."
        w["embed"][:, :2] = 0
        w["embed"][query, 0] = 6.0
        w["embed"][key, 1] = 6.0
        w[p + "q"][:, 0] = 1.0  # the query's direction is e0 only
        w[p + "q"][:, 1:] = 0
        w[p + "dkv"][0] = 0
        w[p + "dkv"][0, 1] = 4.0  # latent 0 carries the key's mark
        w[p + "dkv.norm"][0] = 1.0
        w[p + "uk"][:, 0] = 1.0
        w[p + "uk"][:, 1:] *= 0.02

    return edit


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("window", [2, 33, 64, 65, 130])
def test_keys_just_inside_and_just_outside_the_window(tmp_path, window, path):
    m = Model(tmp_path, [L(window=window, mlp=False, scale=0.25)], path, edit=standing_out())
    for place in (window, window + 1, 127 + window, 128 + window):  # the query's position: edges of pages and batches
        for gap in (window - 1, window):
            ids = ids_of(place + 3, vocab=80)
            ids[place], ids[place - gap] = 90, 91
            want = m.expected(ids)
            if gap > 0:
                wrong = m.expected(ids, ["window-1" if gap == window - 1 else "window+1"])
                assert m.error(want[place : place + 1], wrong[place : place + 1]) > 0.3
            for cuts in ([len(ids)], [place, 1, 2], [place - 1, 2, 2] if place > 1 else [1] * len(ids)):
                m.check(m.run(ids, cuts), want)


@pytest.mark.parametrize("path", PATHS)
def test_far_keys_and_page_borders(tmp_path, path):
    """One key among hundreds, at and around the borders of pages and tiles."""
    m = Model(tmp_path, [L(window=600, mlp=False, scale=0.25), L(window=600, kv_from=0, mlp=False)], path,
              edit=standing_out())
    n = 520
    for key in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 447, 448, 511):
        ids = ids_of(n, vocab=80)
        ids[key], ids[n - 1] = 91, 90
        moved = list(ids)
        moved[key], moved[(key + 1) % (n - 1)] = ids[(key + 1) % (n - 1)], 91
        want = m.expected(ids)
        for cuts in ([n], [n - 1, 1], [300, 219, 1]):
            m.check(m.run(ids, cuts), want)


@pytest.mark.parametrize("path", PATHS)
def test_first_tokens(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    for n in (1, 2, 3, 4):
        ids = ids_of(n, seed=n)
        m.check(m.run(ids), m.expected(ids))
        m.check(m.run(ids, [1] * n), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_rollback_and_beam_reorder(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    pool = m.engine.pool
    ids = ids_of(150)
    seq = pool.open()
    m.run(ids[:120] + ids_of(30, seed=9), sequence=seq)
    (y,) = m.engine.step(m.uids, [StepEntry(seq, m.embed(ids[120:]), 120)])  # back to 120, other tokens
    m.check(y.double().cpu(), m.expected(ids)[120:])
    with pytest.raises(ValueError, match="ahead of the cache"):
        seq.prepare(151, 1)
    seq.close()
    # two hypotheses; both continue the second one with different tokens
    a, b = pool.open(), pool.open()
    m.run(ids_of(70, seed=1), sequence=a)
    m.run(ids[:70], sequence=b)
    pool.reorder([a, b], [1, 1])
    tails = [ids[70:100], ids_of(30, seed=4)]
    outs = [[], []]
    for i in range(30):
        ys = m.engine.step(m.uids, [StepEntry(s, m.embed([t[i]]), 70 + i) for s, t in zip((a, b), tails)])
        for o, y in zip(outs, ys):
            o.append(y)
    for o, t in zip(outs, tails):
        m.check(torch.cat(o).double().cpu(), m.expected(ids[:70] + t)[70:])
    a.close(), b.close()
    assert pool.free_pages == pool.num_pages and not any(pool._refs)


@pytest.mark.parametrize("path", PATHS)
def test_long_steps_are_cut(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    m.engine.max_step_tokens = 50
    ids = [ids_of(130, seed=1), ids_of(20, seed=2), ids_of(45, seed=3)]
    seqs = [m.engine.pool.open() for _ in ids]
    ys = m.engine.step(m.uids, [StepEntry(s, m.embed(t), 0) for s, t in zip(seqs, ids)])
    for y, t in zip(ys, ids):
        m.check(y.double().cpu(), m.expected(t))


@pytest.mark.parametrize("path", PATHS)
def test_stateless_forward_equals_the_cached_one(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = [ids_of(75, seed=1), ids_of(75, seed=2)]
    x = torch.stack([m.embed(t) for t in ids])
    cached = m.engine.forward(m.uids, x)
    shared, plain = {}, x
    for uid in m.uids:
        plain = m.engine.blocks[uid](plain, shared=shared)
    for i, t in enumerate(ids):
        m.check(cached[i].double().cpu(), m.expected(t))
        m.check(plain[i].detach().double().cpu(), m.expected(t))


# ------------------------------------------------------------- pool and batch


def test_pool_limits_and_slots():
    pool = PagedPool({0: 32}, 3, dtype=torch.float32, device="cpu", max_sequences=2)
    a, b = pool.open(), pool.open()
    with pytest.raises(AllocationFailed, match="slots"):
        pool.open()
    a.prepare(0, 65)
    assert len(a.pages) == 2
    with pytest.raises(AllocationFailed):
        b.prepare(0, 65)
    a.advance(65)
    a.prepare(10, 1)  # rolls back into the first page
    assert len(a.pages) == 1 and pool.free_pages == 2
    b.prepare(0, 128)
    b.close()
    b.close()
    a.close()
    assert pool.free_pages == 3 and pool.live_sequences == 0


def test_batch_rows_and_tiles():
    batch = PagedBatch([[4], [2, 0], [1]], [0, 63, 9], [3, 2, 1], torch.device("cpu"))
    assert batch.tokens == 6 and batch.row_ranges() == [(0, 3), (3, 5), (5, 6)] and not batch.decode_only
    assert batch.max_end == 65 and batch.run_tokens(8) == 8 and batch.run_tokens(100) == 1


# --------------------------------------------------------- kernels, one by one


@pytest.mark.gpu
@pytest.mark.parametrize("heads,rank,window,dtype", [
    (1, 32, 0, "bfloat16"), (8, 96, 40, "bfloat16"), (20, 160, 64, "bfloat16"), (70, 512, 100, "bfloat16"),
    (3, 544, 33, "bfloat16"), (5, 64, 50, "float32"),
])
def test_latent_attention_kernel(heads, rank, window, dtype):
    """Every key split agrees with the dense computation, on scattered pages."""
    from petals_amd.ops import latent

    torch.manual_seed(0)
    dt = getattr(torch, dtype)
    starts, lens = [0, 130, 63], [40, 1, 70]
    cache = torch.randn(9, PAGE_SIZE, rank, device="cuda").to(dt)
    pages = [[3], [5, 0, 7], [8, 1, 2]]
    batch = PagedBatch(pages, starts, lens, torch.device("cuda"))
    q = torch.randn(batch.tokens, heads, rank, device="cuda").to(dt)
    scale = 1.5 * rank**-0.5
    want = torch.empty(batch.tokens, heads, rank, dtype=torch.float64)
    for (lo, hi), p, s in zip(batch.row_ranges(), pages, starts):
        c = cache[p].reshape(-1, rank)[: s + hi - lo].double().cpu()
        score = torch.einsum("thr,kr->htk", q[lo:hi].double().cpu(), c) * scale
        seen = oracle.window_mask(len(c), window or len(c))[s:]
        want[lo:hi] = torch.einsum("htk,kr->thr", score.masked_fill(~seen, -float("inf")).softmax(-1), c)
    run = batch.run_tokens(heads)
    for splits in (0, 1, 2, 5):
        got = latent.hip().latent_attention(
            q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, batch.max_end, window, scale, splits
        )
        assert (got.double().cpu() - want).abs().max() < (2e-5 if dtype == "float32" else 3e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("t,experts,top,d", [(1, 1, 1, 7), (3, 8, 2, 128), (70, 300, 9, 1000), (65, 5, 5, 129)])
@pytest.mark.parametrize("slots", [0, 3])
def test_sublayer_out_kernel(t, experts, top, d, slots):
    from petals_amd.ops import latent

    torch.manual_seed(0)
    dp = -(-d // 128) * 128
    y = torch.randn(t * max(slots, 1), dp, device="cuda")
    sw = torch.rand(t, slots, device="cuda") if slots else None
    w, x = torch.randn(d, device="cuda") * 0.3, torch.zeros(t, dp, device="cuda")
    x[:, :d] = torch.randn(t, d, device="cuda")
    router = torch.zeros(experts, dp, device="cuda")
    router[:, :d] = torch.randn(experts, d, device="cuda")
    xo, xb, sel, sw_out = latent.hip().sublayer_out(y, sw, w, 1e-5, x, dp, True, router, top)
    s = (y.view(t, -1, dp).double() * (sw[..., None].double() if slots else 1)).sum(1)[:, :d].cpu()
    want = x[:, :d].double().cpu() + oracle.zero_centered_norm(s, w.double().cpu(), 1e-5)
    assert (xo[:, :d].double().cpu() - want).abs().max() < 1e-4 and (xo[:, d:] == 0).all()
    assert torch.equal(xb, xo.bfloat16())
    scores, _ = oracle.route(xo[:, :d].double().cpu(), router[:, :d].double().cpu(), top)
    p = torch.softmax(xo[:, :d].double() @ router[:, :d].double().T, -1).cpu()
    assert (sw_out.double().cpu() - scores).abs().max() < 1e-5
    assert (p.gather(1, sel.long().cpu()) - scores).abs().max() < 1e-5
    assert all(len(set(r)) == top for r in sel.tolist())


@pytest.mark.gpu
@pytest.mark.parametrize("pairs,experts", [(1, 1), (5, 64), (4000, 7), (33, 2), (2048, 300)])
def test_moe_group_kernel(pairs, experts):
    from petals_amd.ops import latent

    sel = torch.randint(0, experts, (pairs,), dtype=torch.int32)
    order, tiles = (t.cpu() for t in latent.hip().moe_group(sel.cuda(), experts, 32))
    assert sorted(order[order >= 0].tolist()) == list(range(pairs))
    for i, e in enumerate(tiles.tolist()):
        rows = order[32 * i : 32 * i + 32]
        rows = rows[rows >= 0].long()
        assert (sel[rows] == e).all() and (len(rows) > 0) == (e >= 0)


@pytest.mark.gpu
@pytest.mark.parametrize("t,h,k,n", [(1, 3, 32, 40), (16, 2, 96, 130), (17, 1, 45, 33), (200, 4, 128, 96)])
@pytest.mark.parametrize("a_dtype", ["float32", "bfloat16"])
def test_batched_linear_kernel(t, h, k, n, a_dtype):
    from petals_amd.ops import latent

    torch.manual_seed(0)
    a = torch.randn(t, h * k + 8, device="cuda").to(getattr(torch, a_dtype))[:, : h * k].view(t, h, k)
    w = torch.randn(h, n, k, device="cuda")
    for wd in ("bfloat16", "float32")[: 2 if a_dtype == "float32" else 1]:
        wt = w.to(getattr(torch, wd))
        got = latent.hip().batched_linear(a, wt, True).double().cpu()
        exact = a.to(wt.dtype).double().cpu().transpose(0, 1) @ wt.double().cpu().transpose(1, 2)
        assert (got - exact.transpose(0, 1)).abs().max() < 1e-3


@pytest.mark.gpu
def test_decode_graph_replays_match_eager(tmp_path, monkeypatch):
    """Replays with other work between them, requests coming and going."""
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
        m.check(a.double().cpu(), b.double().cpu(), slack=0.5)
