"""Soselix against its plain oracle (tests/soselix_oracle.py): mechanisms alone, and
whole models through the span engine that serves them - prompts, portions, decoding,
mixed batches, pages and state slots used again - on the CPU path and, marked gpu, on
the HIP kernels in float32 and bfloat16."""

import math
import random

import pytest
import torch

import soselix_oracle as oracle
from petals_amd.models.config_base import load_model_config
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

L, H, M = oracle.latent_layer, oracle.hgrn_layer, oracle.mamba_layer
SHAPES = {
    # every kind of layer with and without a feed-forward; two caches, each read by another layer
    "mixed": [
        H(heads=4, dim=12, vdim=20, ff=30), L(heads=6, dim=16, vdim=12, kv_rank=40, rot_dim=8),
        M(heads=4, vdim=12, state=20, groups=2, norm_groups=3, ff=None),
        L(heads=3, dim=24, vdim=20, kv_rank=40, rot_dim=8, q_rank=7, kv_from=1, ff=None, scale=0.3),
        L(heads=4, dim=8, vdim=16, kv_rank=24, rot_dim=6, base=90.0, ff=40),
        H(heads=2, dim=16, vdim=16), M(heads=6, vdim=8, state=16, groups=3, conv=2, norm_groups=6),
        L(heads=5, dim=40, vdim=4, kv_rank=24, rot_dim=6, base=90.0, kv_from=4),
    ],
    # everything that can be one is one
    "ones": [
        H(heads=1, dim=1, vdim=1, ff=1), M(heads=1, vdim=1, state=1, groups=1, conv=1, norm_groups=1, ff=1),
        L(heads=1, dim=1, vdim=1, kv_rank=2, q_rank=2, rot_dim=2, ff=1),
        L(heads=1, dim=1, vdim=1, kv_rank=2, q_rank=2, rot_dim=2, ff=1, kv_from=2),
    ],
    # equal sizes everywhere
    "equal": [
        H(heads=32, dim=32, vdim=32, ff=32), M(heads=32, vdim=32, state=32, groups=32, conv=4, norm_groups=32, ff=32),
        L(heads=32, dim=32, vdim=32, kv_rank=32, q_rank=32, rot_dim=32, ff=32),
    ],
    # head counts and sizes that are no multiple of anything, more heads than a tile has rows
    "wide": [
        H(heads=5, dim=70, vdim=133), L(heads=72, dim=33, vdim=65, kv_rank=131, rot_dim=34, q_rank=51),
        M(heads=21, vdim=35, state=75, groups=1, conv=5, norm_groups=7),
        M(heads=34, vdim=16, state=8, groups=2, conv=3, norm_groups=1),
        L(heads=9, dim=72, vdim=40, kv_rank=200, rot_dim=66),
    ],
    # beyond the tiled kernels' sizes
    "long_heads": [
        L(heads=2, dim=24, vdim=270, kv_rank=530, rot_dim=70), H(heads=2, dim=270, vdim=270),
        M(heads=1, vdim=2100, state=24, groups=1, norm_groups=1), L(heads=3, dim=150, vdim=24, kv_rank=500, rot_dim=80),
    ],
    "no_attention": [H(), M(groups=1), H(heads=1)],
    "no_recurrence": [L(), L(kv_from=0), L(heads=3, kv_rank=64, rot_dim=64)],
}


class Model:
    """A random model served by a SpanEngine, and its oracle. (A norm over few values that
    happen to be small amplifies bf16 rounding without bound if eps is tiny.)"""

    def __init__(self, tmp_path, layers, path=("cpu", "float32"), *, width=40, vocab=97, tokens=1024, seed=0, edit=None,
                 eps=1e-2, sequences=None, mult=0.6):
        self.device, self.dtype = path
        self.raw = oracle.config_dict(vocab=vocab, width=width, layers=layers, eps=eps, mult=mult)
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
        return self.weights["embed"][torch.as_tensor(ids)].float().to(self.device) * self.raw["embedding"]["scale"]

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
def test_rotate_halves(n, dims):
    x = torch.randn(70, 3, n, dtype=F64)
    got = reference.rotate_halves(x, torch.arange(70)[:, None], dims, 30.0)
    assert (got - oracle.rotate(x, torch.arange(70), dims, 30.0)).abs().max() < 1e-6
    # a turn keeps lengths, and scores depend on distances only
    assert torch.allclose(got.norm(dim=-1), x.norm(dim=-1), rtol=1e-6)
    q, k = x[:1].expand(2, 3, n), x[1:2].expand(2, 3, n)
    y = reference.rotate_halves(q, torch.tensor([[40], [7]]), dims, 30.0)
    z = reference.rotate_halves(k, torch.tensor([[43], [10]]), dims, 30.0)
    assert torch.allclose((y * z).sum(-1)[0], (y * z).sum(-1)[1], atol=1e-5)


def test_forget_gate_keeps_small_writes():
    z = torch.tensor([-90.0, -20.0, -1.0, 0.0, 2.0, 16.0, 30.0])
    for lower in (0.0, 0.4, 0.97):
        k, f = reference.forget_gate(z, torch.full_like(z, lower))
        want = oracle.forget_gate(z.double(), lower)
        assert torch.allclose(f.double(), want, rtol=1e-6, atol=1e-30)
        exact = (1 - lower) / (1 + torch.exp(z.double()))
        assert torch.allclose(k.double(), exact, rtol=1e-5, atol=1e-30)


@pytest.mark.parametrize("per_channel", [True, False])
def test_gated_linear_attention_and_its_state(per_channel):
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(1, 30, 3, n, generator=g, dtype=F64) for n in (5, 5, 4))
    decay = torch.rand(1, 30, 3, 5 if per_channel else 1, generator=g, dtype=F64)
    want = oracle.decay_recurrence(q[0], k[0], v[0], decay[0].expand(30, 3, 5))
    whole, last = reference.gated_linear_attention(q, k, v, decay, torch.zeros(1, 3, 5, 4, dtype=F64))
    assert (whole[0] - want).abs().max() < 1e-9
    state, parts = torch.zeros(1, 3, 5, 4, dtype=F64), []
    for lo, hi in ((0, 1), (1, 13), (13, 30)):
        o, state = reference.gated_linear_attention(*(t[:, lo:hi] for t in (q, k, v, decay)), state)
        parts.append(o)
    assert (torch.cat(parts, 1) - whole).abs().max() < 1e-9 and (state - last).abs().max() < 1e-9


@pytest.mark.parametrize("groups", [1, 2, 6])
def test_group_norm(groups):
    x, w = torch.randn(7, 12), torch.randn(12)
    want = oracle.group_norm(x.double(), w.double(), groups, 1e-3)
    assert (reference.group_rms_norm(x, w, groups, 1e-3).double() - want).abs().max() < 1e-5


def test_xielu_on_both_sides_of_zero():
    z = torch.tensor([-60.0, -3.0, -0.5, -1e-3, 0.0, 1e-3, 0.7, 9.0])
    p, q = torch.tensor(-0.3), torch.tensor(1.1)
    want = oracle.xielu(z.double(), p.double(), q.double())
    assert torch.allclose(reference.xielu(z, p, q).double(), want, rtol=1e-5, atol=1e-8)


def test_config_reads_every_layer_and_rejects_nonsense(tmp_path):
    import copy
    import json

    raw = oracle.config_dict(layers=SHAPES["mixed"], width=24, mult=0.31, scale=2.5, eps=3e-5)
    oracle.save_model(str(tmp_path), raw, {"x": torch.zeros(1)})
    c = load_model_config(str(tmp_path))
    assert (c.num_blocks, c.hidden_size, c.layer_norm_eps, c.residual_mult, c.embedding_scale) == (8, 24, 3e-5, 0.31, 2.5)
    m = c.spec(4).mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.rot_base, m.scale) == (4, 8, 6, 16, 24, 90.0, 0.2)
    assert c.spec(3).mlp is None and c.spec(3).mixer.kv_from == 1 and c.spec(0).mlp.ff == 30
    assert sorted(c.valid_cuts()) == [0, 1, 4, 8] and not c.rewindable
    assert c.cache_values_per_token(1) == 64 + 32 and c.cache_values_per_token(3) == c.cache_values_per_token(0) == 0
    assert c.state_shapes(0) == {"matrix": (4, 16, 32)} and c.state_shapes(1) == {}
    assert c.state_shapes(6) == {"matrix": (6, 16, 16), "conv": (2, 48 + 2 * 3 * 16)}

    def broken(change):
        d = copy.deepcopy(raw)
        change(d["layers"])
        (tmp_path / "config.json").write_text(json.dumps(d))
        with pytest.raises((ValueError, KeyError)):
            load_model_config(str(tmp_path))

    broken(lambda l: l[0].update(type="attention"))
    broken(lambda l: l[2]["mixer"].update(groups=3))
    broken(lambda l: l[2]["mixer"].update(norm_groups=5))
    broken(lambda l: l[3]["mixer"].update(kv_from=2))
    broken(lambda l: l[3]["mixer"].update(kv_from=3))
    broken(lambda l: l[3]["mixer"].update(kv_rank=48))
    broken(lambda l: l[7]["mixer"].update(kv_from=3))  # which has no latent of its own
    broken(lambda l: l[0]["mlp"].update(kind="experts"))
    broken(lambda l: l[1]["mixer"].update(heads=2.5))


def test_loader_refuses_incomplete_checkpoints(tmp_path):
    raw = oracle.config_dict(layers=SHAPES["mixed"])
    for name, change in (("l0.mix.lower", None), ("l1.mix.sink", None), ("l2.mix.conv", lambda t: t[:, 1:]),
                         ("l3.mix.uk", lambda t: t[1:]), ("l4.mlp.act", lambda t: t[:1])):
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
@pytest.mark.parametrize("width,vocab,eps,mult", [(8, 11, 1e-6, 1.0), (131, 40, 1e-3, 0.25), (256, 300, 0.3, 1.7)])
def test_other_widths_and_constants(tmp_path, width, vocab, eps, mult, path):
    m = Model(tmp_path, SHAPES["mixed"], path, width=width, vocab=vocab, eps=eps, seed=3, mult=mult)
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
        "no_rotation", "rotate_neighbours", "no_sink", "forgets_far", "no_gate", "lost_state", "read_before_write",
        "no_lower", "write_all", "no_conv_bias", "conv_one_less", "group_interleave", "dt_clamp", "no_skip",
        "gate_after", "one_norm", "act_half",
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


def standing_out(rotated, query=90, key=91):
    """Weights under which token `query` scores far higher on token `key` than on any
    other, through the latent's part of the score or through the rotated one."""

    def edit(w):
        p = "l0.mix."
        w["embed"][:, :2] = 0
        w["embed"][query, 0] = 6.0
        w["embed"][key, 1] = 6.0
        rank = w[p + "uk"].shape[1]
        w[p + "dq"][:] = 0
        w[p + "dq"][0, 0] = 1.0  # the query latent of other tokens is zero
        w[p + "dq.norm"][:] = 1.0
        w[p + "dkv"][:, 1] = 0
        w[p + "uq"][:] = 0
        w[p + "uk"][:] = 0
        dim, per = w[p + "uk"].shape[0], w[p + "uq"].shape[0]
        heads = w[p + "sink"].shape[0]
        uq = w[p + "uq"].view(heads, per // heads, -1)
        if rotated:
            w[p + "dkv"][rank:] = 0
            w[p + "dkv"][rank, 1] = 2.0
            uq[:, dim // heads, 0] = 1.5
        else:
            w[p + "dkv"][0] = 0
            w[p + "dkv"][0, 1] = 2.0
            w[p + "uk"][:, 0] = 0.6
            uq[:, : dim // heads, 0] = 0.5

    return edit


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("heads,rotated", [(1, False), (17, False), (2, True)])
def test_far_keys_and_page_borders(tmp_path, path, heads, rotated):
    """One key among hundreds, at and around the borders of pages and tiles."""
    # slow turns, so that a far key's rotated part still points its way
    layer = L(heads=heads, dim=16, vdim=16, kv_rank=32, q_rank=16, rot_dim=2, base=10.0, ff=None, scale=0.5)
    m = Model(tmp_path, [layer], path, edit=standing_out(rotated))
    n = 520
    keys = (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 447, 448, 511)[:: 1 if heads == 1 else 3]
    if rotated:  # a pair that turns by one radian a position: distances near whole turns
        keys = (n - 1 - 6, n - 1 - 44, n - 1 - 201, n - 1 - 509)
    for key in keys:
        ids = ids_of(n, vocab=80)
        ids[key], ids[n - 1] = 91, 90
        want = m.expected(ids)
        assert m.error(want[-1:], m.expected(ids[:key] + [5] + ids[key + 1 :])[-1:]) > 0.1  # without that key
        for cuts in ([n], [n - 1, 1], [300, 219, 1]):
            m.check(m.run(ids, cuts), want)


def slow_decay(w):
    for name, t in w.items():
        if name.endswith("A_log"):
            t.fill_(-9.0)
        if name.endswith("lower"):
            t.fill_(0.996)


@pytest.mark.parametrize("path", PATHS)
@pytest.mark.parametrize("layer", [H(heads=4, dim=32, vdim=16), M(heads=4, vdim=16, state=32, groups=2, norm_groups=4, ff=None)],
                         ids=["hgrn2", "mamba2"])
def test_state_remembers_the_first_token(tmp_path, layer, path):
    """Decays close to one: the first token still shows hundreds of tokens later,
    however the tokens between are cut."""
    m = Model(tmp_path, [layer], path, edit=slow_decay)
    pair = [ids_of(260, vocab=3, seed=7), None]
    pair[1] = [96] + pair[0][1:]
    wants = [m.expected(ids) for ids in pair]
    late = m.errors(wants[0][-40:], wants[1][-40:])
    assert float(late.mean()) > 10 * TOLERANCE["float32"]
    for ids, want in zip(pair, wants):
        for cuts in ([260], [1] * 20 + [240], [100, 2, 3, 16, 129] + [1] * 10):
            m.check(m.run(ids, cuts), want, slack=0.3)


@pytest.mark.parametrize("path", PATHS)
def test_strong_decays_do_not_overflow(tmp_path, path):
    def edit(w):
        w["l0.mix.A_log"][:] = torch.tensor([5.0, -2.0, 3.0, 1.0])
        w["l0.mix.dt_bias"][:] = torch.tensor([4.0, -30.0, 0.0, 2.0])
        w["l1.mix.f.b"][:] = torch.tensor([-100.0, -9.0, 0.0, 100.0]).repeat(24)
        w["l1.mix.lower"][::3] = 0

    m = Model(tmp_path, [M(heads=4, vdim=16, state=32, groups=2, norm_groups=4), H(heads=3, dim=32, vdim=16)], path, edit=edit)
    ids = ids_of(100)
    m.check(m.run(ids), m.expected(ids))
    m.check(m.run(ids, [37] + [1] * 10 + [53]), m.expected(ids))


@pytest.mark.parametrize("path", PATHS)
def test_sink_and_gate_take_their_share_of_a_single_key(tmp_path, path):
    def edit(w):
        w["l0.mix.sink"][:] = torch.tensor([9.0, -60.0, 0.0, 80.0])
        w["l0.mix.g"] *= 3

    m = Model(tmp_path, [L(heads=4, ff=None)], path, edit=edit)
    for ids in ([5], ids_of(70)):
        want = m.expected(ids)
        assert m.error(want, m.expected(ids, ["no_sink"])) > 0.1 and m.error(want, m.expected(ids, ["no_gate"])) > 0.1
        m.check(m.run(ids), want)
        m.check(m.run(ids, [1] * len(ids)), want)


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


@pytest.mark.parametrize("path", PATHS[:2])
def test_chains_cut_where_no_cache_is_shared(tmp_path, path):
    """The span in two engines, as two servers would run it."""
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = ids_of(60)
    for cut in (1, 4):
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
    with pytest.raises(ValueError, match="reads the cache"):
        m.engine.check_chain(m.uids[2:])


@pytest.mark.parametrize("path", PATHS)
def test_stateless_forward_equals_the_cached_one(tmp_path, path):
    m = Model(tmp_path, SHAPES["mixed"], path)
    ids = [ids_of(75, seed=1), ids_of(75, seed=2)]
    x = torch.stack([m.embed(t) for t in ids])
    cached, plain, shared = m.engine.forward(m.uids, x), x, {}
    for uid in m.uids:
        plain = m.engine.blocks[uid](plain, shared=shared)
    for i, t in enumerate(ids):
        m.check(m.residual(cached[i]), m.expected(t))
        m.check(m.residual(plain[i]), m.expected(t))


# --------------------------------------------------------- kernels, one by one


@pytest.mark.gpu
@pytest.mark.parametrize("heads,rank,rot,dtype", [
    (1, 32, 32, "bfloat16"), (8, 32, 64, "bfloat16"), (12, 128, 32, "bfloat16"), (70, 96, 32, "bfloat16"),
    (5, 160, 96, "bfloat16"), (32, 256, 64, "bfloat16"), (6, 384, 64, "bfloat16"), (40, 512, 64, "bfloat16"),
    (3, 544, 32, "bfloat16"), (6, 64, 32, "float32"),
])
def test_latent_attention_kernel(heads, rank, rot, dtype):
    """Every key split and row layout agrees with the dense computation, on scattered
    pages; with and without a sink and a factor per head."""
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    dt = getattr(torch, dtype)
    scale, width = 1.5 * (rank + rot) ** -0.5, rank + rot
    cache = torch.randn(9, PAGE_SIZE, width, device="cuda").to(dt)
    for starts, lens in (([0, 130, 63], [40, 1, 70]), ([0, 130, 63], [1, 1, 1])):
        pages = [[3], [5, 0, 7], [8, 1, 2]]
        batch = PagedBatch(pages, starts, lens, torch.device("cuda"))
        q = torch.randn(batch.tokens, heads, width, device="cuda").to(dt)
        sink, factor = 3 * torch.randn(heads, device="cuda"), torch.rand(batch.tokens, heads, device="cuda")
        run = batch.run_tokens(heads)
        for sink_, factor_ in ((sink, factor), (None, None)):
            want = torch.empty(batch.tokens, heads, rank, dtype=F64)
            for (lo, hi), p, s in zip(batch.row_ranges(), pages, starts):
                rows = cache[p].reshape(-1, width)[: s + hi - lo].double().cpu()
                unseen = torch.arange(len(rows))[s:, None] < torch.arange(len(rows))[None, :]
                for n in range(heads):
                    score = (q[lo:hi, n].double().cpu() @ rows.T * scale).masked_fill(unseen, -math.inf)
                    p_ = oracle.sink_softmax(score, sink[n].double().cpu(), () if sink_ is not None else ("no_sink",))
                    want[lo:hi, n] = p_ @ rows[:, :rank]
            if factor_ is not None:
                want *= factor.double().cpu()[:, :, None]
            for splits in (0, 1, 2, 5):
                got = recurrent.hip().latent_attention(
                    q, cache, batch.pos, batch.owner, batch.tables, batch.tiles(run), run, batch.max_end, 0, scale,
                    splits, rank, sink_, factor_,
                )
                assert got.shape == (batch.tokens, heads, rank)
                assert (got.double().cpu() - want).abs().max() < (2e-5 if dtype == "float32" else 3e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("q_rank,kv_rank,rot,turned,heads", [(24, 40, 8, 8, 6), (1, 1, 2, 2, 1), (600, 300, 40, 20, 33)])
def test_latent_rows_and_rotation_at_any_position(q_rank, kv_rank, rot, turned, heads, dtype):
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    hip, dt, eps, base = recurrent.hip(), getattr(torch, dtype), 1e-4, 3000.0
    lp, rp, qp = (-(-n // k) * k for n, k in ((kv_rank, 32), (rot, 32), (q_rank, 8)))
    i = torch.arange(turned // 2, dtype=F64)
    quarters = (base ** (-2 * i / turned) * 2 / math.pi).cuda()
    starts, lens = [0, 4000, 1_000_001], [20, 1, 70]
    pages = [[3], [0] * 62 + [5], [0] * 15625 + [8, 1]]
    batch = PagedBatch(pages, starts, lens, torch.device("cuda"))
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)])
    y = torch.randn(batch.tokens, 5 + q_rank + kv_rank + rot + heads, device="cuda").to(dt)
    at_q, at_kv, at_g = 5, 5 + q_rank, 5 + q_rank + kv_rank + rot
    w_q, w_kv = torch.randn(q_rank, device="cuda"), torch.randn(kv_rank, device="cuda")
    cache = torch.full((9, PAGE_SIZE, lp + rp), 7.0, device="cuda", dtype=dt)
    cq, gate = hip.latent_rows(y, at_q, w_q, qp, True, at_kv, w_kv, lp, rot, quarters, cache, at_g, heads, batch.pos,
                               batch.owner, batch.tables, eps)
    yd, tol = y.double().cpu(), 1e-5 if dtype == "float32" else 2e-2
    want = oracle.norm(yd[:, at_q:at_kv], w_q.double().cpu(), eps)
    assert (cq[:, :q_rank].double().cpu() - want).abs().max() < 1e-4 and (cq[:, q_rank:] == 0).all()
    assert (gate.double().cpu() - torch.sigmoid(yd[:, at_g:])).abs().max() < 1e-5
    rows = torch.cat([cache[torch.tensor(p)[torch.arange(s, s + n) // 64], torch.arange(s, s + n) % 64]
                      for p, s, n in zip(pages, starts, lens)]).double().cpu()
    c = oracle.norm(yd[:, at_kv : at_kv + kv_rank], w_kv.double().cpu(), eps)
    k = oracle.rotate(yd[:, at_kv + kv_rank : at_g], pos, turned, base)
    assert (rows[:, :kv_rank] - c).abs().max() < tol * 5 and (rows[:, lp : lp + rot] - k).abs().max() < tol * 5
    assert (rows[:, kv_rank:lp] == 0).all() and (rows[:, lp + rot :] == 0).all()
    assert int((cache != 7.0).any(-1).sum()) == batch.tokens  # and no other row
    # a layer that reads another's cache writes none
    before = cache.clone()
    hip.latent_rows(y, at_q, w_q, qp, True, -1, None, lp, rot, quarters, cache, at_g, heads, batch.pos, batch.owner,
                    batch.tables, eps)
    assert torch.equal(cache, before)
    qs = torch.randn(batch.tokens, 3 + heads * rp, device="cuda").to(dt)
    q = torch.full((batch.tokens, heads, lp + rp), 7.0, device="cuda", dtype=dt)
    hip.rotate_queries(qs, 3, rp, quarters, batch.pos, q, lp)
    want = oracle.rotate(qs[:, 3:].double().cpu().view(-1, heads, rp), pos, turned, base)
    assert (q[:, :, lp:].double().cpu() - want).abs().max() < tol * 5 and (q[:, :, :lp] == 7.0).all()


def run_ragged(total, tail, slots, prefill, decode, wants, tol):
    """Portions of four sequences, then single tokens, in scattered slots."""
    starts = [0] * 4

    def rel(got, want):
        return float((got.double().cpu() - want).abs().max() / want.abs().max())

    for counts in ([20, 1, 2, 50], [17, 0, 14, 0]):
        live = [i for i in range(4) if counts[i]]
        b = PagedBatch([[0]] * len(live), [starts[i] for i in live], [counts[i] for i in live], torch.device("cuda"),
                       [slots[i] for i in live])
        out = prefill(b, live, [(starts[i], starts[i] + counts[i]) for i in live])
        for i, (lo, hi) in zip(live, b.row_ranges()):
            assert rel(out[lo:hi], wants[i][starts[i] : starts[i] + hi - lo]) < tol
            starts[i] += hi - lo
    assert starts == [n - tail for n in total]
    for _ in range(tail if decode else 0):
        b = PagedBatch([[0]] * 4, starts, [1] * 4, torch.device("cuda"), slots)
        out = decode(b, range(4), [(s, s + 1) for s in starts])
        for i in range(4):
            assert rel(out[i], wants[i][starts[i]]) < tol
            starts[i] += 1


def used_state(slots, *shape, dim, vdim):
    """What a slot's last user left; padding stays zero in a pool's life."""
    state = torch.full((7, *shape), 9.0, device="cuda")
    for s in slots:
        state[s, :, dim:] = 0
        state[s, :, :, vdim:] = 0
    return state


TOTAL, TAIL, SLOTS = [42, 6, 21, 55], 5, [5, 0, 3, 1]


@pytest.mark.gpu
@pytest.mark.parametrize("heads,dim,vdim", [(1, 1, 1), (3, 12, 20), (10, 64, 64), (4, 128, 128), (2, 200, 48), (2, 16, 300),
                                            (64, 32, 32), (1, 500, 2064)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_forget_gate_kernels(heads, dim, vdim, dtype):
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    hip, dt, eps = recurrent.hip(), getattr(torch, dtype), 1e-5
    n, gap = heads * dim, 8 if dim % 8 == 0 else 3  # aligned columns and others
    cols = [0, n + gap, 2 * n + gap]
    width = -(-(cols[2] + heads * vdim) // 8) * 8
    ys = [torch.randn(t, width).to(dt) for t in TOTAL]
    bias, lower, norm_w = 2 * torch.randn(n), torch.rand(n), 1 + 0.3 * torch.randn(vdim)
    lower[::3] = 0
    wants, raws = [], []
    for y in ys:
        q, f, v = (y.double()[:, c : c + k] for c, k in zip(cols, (n, n, heads * vdim)))
        f = oracle.forget_gate(f + bias.double(), lower.double()).view(-1, heads, dim)
        o = oracle.decay_recurrence(oracle.silu(q).view(-1, heads, dim), 1 - f, v.reshape(-1, heads, vdim), f)
        raws.append(o.flatten(1))
        wants.append(oracle.norm(o, norm_w.double(), eps).flatten(1))
    state = used_state(SLOTS, heads, -(-dim // 16) * 16, -(-vdim // 16) * 16, dim=dim, vdim=vdim)
    bias, lower, norm_w = bias.cuda(), lower.cuda(), norm_w.cuda()

    def rows(live, ranges):
        return torch.cat([ys[i][lo:hi] for i, (lo, hi) in zip(live, ranges)]).cuda()

    def prefill(b, live, ranges):
        o = hip.forget_prefill(rows(live, ranges), bias, lower, b.tiles(16), b.chunk_bounds(16), b.pos, b.owner, b.slot,
                               state, heads, dim, vdim, cols)
        want = torch.cat([raws[i][lo:hi] for i, (lo, hi) in zip(live, ranges)])
        assert (o.double().cpu() - want).abs().max() < 1e-4 * want.abs().max()
        return hip.group_norm(o, None, norm_w, heads, heads * vdim, True, eps)

    def decode(b, live, ranges):
        out = hip.forget_decode(rows(live, ranges), bias, lower, norm_w, b.pos, b.slot, state, heads, dim, vdim, cols,
                                heads * vdim + 8, eps)
        assert (out[:, heads * vdim :] == 0).all() and out.dtype == dt
        return out[:, : heads * vdim]

    run_ragged(TOTAL, TAIL, SLOTS, prefill, decode if hip.linear_decodes(dim, vdim) else None, wants,
               5e-4 if dtype == "float32" else 3e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("heads,groups,state,vdim,taps,parts", [
    (1, 1, 1, 1, 1, 1), (4, 2, 20, 12, 4, 3), (40, 1, 64, 64, 4, 1), (6, 6, 128, 64, 3, 2), (34, 2, 16, 16, 5, 17),
    (3, 1, 300, 40, 2, 3), (64, 8, 32, 32, 4, 8),
])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_state_space_kernels(heads, groups, state, vdim, taps, parts, dtype):
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    hip, dt, eps = recurrent.hip(), getattr(torch, dtype), 1e-5
    inner, channels = heads * vdim, heads * vdim + 2 * groups * state
    at_conv = inner if inner % 8 else inner + 8
    at_dt = at_conv + channels
    ys = [torch.randn(t, -(-(at_dt + heads) // 8) * 8).to(dt) for t in TOTAL]
    conv_w, conv_b = torch.randn(channels, taps), 0.3 * torch.randn(channels)
    a_log, dt_bias, skip, norm_w = torch.randn(heads), torch.randn(heads) - 1, torch.randn(heads), torch.randn(inner)
    of = torch.arange(heads) // (heads // groups)
    wants, raws = [], []
    for y in ys:
        y = y.double()
        mixed = oracle.silu(oracle.short_conv(y[:, at_conv:at_dt], conv_w.double(), conv_b.double()))
        x, b, c = mixed.split([inner, groups * state, groups * state], dim=-1)
        x, b, c = x.view(-1, heads, vdim), b.reshape(-1, groups, state)[:, of], c.reshape(-1, groups, state)[:, of]
        step = oracle.softplus(y[:, at_dt : at_dt + heads] + dt_bias.double())
        decay = torch.exp(-torch.exp(a_log.double()) * step)[:, :, None].expand(-1, -1, state)
        o = oracle.decay_recurrence(c, b, step[:, :, None] * x, decay) + skip.double()[:, None] * x
        raws.append(o.flatten(1))
        wants.append(oracle.group_norm(o.flatten(1) * oracle.silu(y[:, :inner]), norm_w.double(), parts, eps))
    matrix = used_state(SLOTS, heads, -(-state // 16) * 16, -(-vdim // 16) * 16, dim=state, vdim=vdim)
    conv = torch.full((7, taps, channels), 9.0, device="cuda")
    weights = [t.cuda() for t in (conv_w.t().contiguous(), conv_b, a_log.exp(), dt_bias, skip)]
    sizes = (matrix, conv, heads, groups, state, vdim, at_conv, at_dt)
    norm_w = norm_w.cuda()

    def normed(o, y, live, ranges):
        want = torch.cat([raws[i][lo:hi] for i, (lo, hi) in zip(live, ranges)])
        assert (o.double().cpu() - want).abs().max() < 1e-4 * want.abs().max()
        out = hip.group_norm(o, y[:, :inner], norm_w, parts, inner + 3, dtype == "float32", eps)
        assert (out[:, inner:] == 0).all()
        return out[:, :inner]

    def rows(live, ranges):
        return torch.cat([ys[i][lo:hi] for i, (lo, hi) in zip(live, ranges)]).cuda()

    def prefill(b, live, ranges):
        y = rows(live, ranges)
        o = hip.ssm_prefill(y, *weights, b.tiles(16), b.chunk_bounds(16), b.pos, b.owner, b.slot, *sizes)
        return normed(o, y, live, ranges)

    def decode(b, live, ranges):
        y = rows(live, ranges)
        return normed(hip.ssm_decode(y, *weights, b.pos, b.slot, *sizes), y, live, ranges)

    run_ragged(TOTAL, TAIL, SLOTS, prefill, decode if hip.linear_decodes(state, vdim) else None, wants,
               5e-4 if dtype == "float32" else 3e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("t,groups,size,shared", [(1, 1, 5, False), (70, 6, 128, True), (9, 3, 500, False), (40, 2, 4100, False)])
def test_group_norm_kernel(t, groups, size, shared):
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    o, w = torch.randn(t, groups * size, device="cuda"), torch.randn(size if shared else groups * size, device="cuda")
    for gate in (None, torch.randn(t, groups * size + 1, device="cuda")[:, 1:], torch.randn_like(o).bfloat16()):
        want = o.double() if gate is None else o.double() * oracle.silu(gate.double())
        want = oracle.group_norm(want, (w.repeat(groups) if shared else w).double(), groups, 1e-2)
        for f32 in (True, False):
            got = recurrent.hip().group_norm(o, gate, w, groups, groups * size, f32, 1e-2)
            assert got.dtype == (torch.float32 if f32 else torch.bfloat16)
            assert (got.double() - want).abs().max() < (1e-4 if f32 else 1e-2) * want.abs().max()


@pytest.mark.gpu
@pytest.mark.parametrize("t,d", [(1, 8), (5, 1000), (300, 264)])
def test_activation_and_scaled_residual_kernels(t, d):
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    hip = recurrent.hip()
    y, b, x0 = 4 * torch.randn(t, d, device="cuda"), torch.randn(d, device="cuda"), torch.randn(t, d, device="cuda")
    p, q = torch.tensor(0.7, dtype=F64), torch.tensor(-0.4, dtype=F64)
    constants = (float(oracle.softplus(p)), 0.5 + float(oracle.softplus(q)))
    y[:, ::2] *= 1e-3
    b[::2] *= 1e-3
    want = oracle.xielu(y.double().cpu() + b.double().cpu(), p, q).cuda()
    got = hip.bias_xielu(y.clone(), b, *constants).double()
    assert ((got - want).abs() / (want.abs() + 1e-3)).max() < 1e-4
    assert (hip.bias_xielu(y.bfloat16(), b, *constants).double() - want).abs().max() < 2e-2 * want.abs().max()
    parts = torch.randn(37, t, d, device="cuda")
    if t <= 8:
        want = oracle.xielu((parts.double().sum(0) + b.double()).cpu(), p, q).cuda()
        assert (hip.bias_xielu(parts, b, *constants).double() - want).abs().max() < 1e-4 * want.abs().max()
        x = x0.clone()
        hip.residual_sum(parts, b, x, d, 0.3)
        assert (x.double() - x0.double() - 0.3 * (parts.double().sum(0) + b.double())).abs().max() < 1e-4
    for bias in (None, b):
        x = x0.clone()
        h = hip.residual_norm(x, y, bias, b, d, 1e-3, True, 0.3)
        want = x0.double() + 0.3 * (y.double() + (0 if bias is None else b.double()))
        assert (x.double() - want).abs().max() < 1e-5
        assert (h[:, :d].double() - oracle.norm(want, b.double(), 1e-3)).abs().max() < 1e-4


@pytest.mark.gpu
@pytest.mark.parametrize("t", [3, 70])
def test_batched_linear_into_a_view(t):
    from petals_amd.ops import recurrent

    torch.manual_seed(0)
    a, w = torch.randn(t, 5, 32, device="cuda"), torch.randn(5, 48, 32, device="cuda")
    for dt, out_dt in ((torch.bfloat16, torch.bfloat16), (torch.bfloat16, torch.float32), (torch.float32, torch.float32)):
        out = torch.full((t, 5, 100), 7.0, device="cuda", dtype=out_dt)
        recurrent.hip().batched_linear(a.to(dt), w.to(dt), out_dt == torch.float32, out[:, :, 3:51])
        want = torch.stack([a[:, h].to(dt).double() @ w[h].to(dt).double().T for h in range(5)], 1)
        assert (out[:, :, 3:51].double() - want).abs().max() < 2e-2 * want.abs().max()
        assert (out[:, :, :3] == 7.0).all() and (out[:, :, 51:] == 7.0).all()


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
