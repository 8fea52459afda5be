"""Rarutar on the GPU against the float64 restatement in tests/rarutar_ref.py (which processes whole sequences, with no cache, no state and no
batching): every mechanism alone, prompts against token-by-token decoding, portions down to two tokens, mixed batches, cells and state slots that are
used again, keys made loud on purpose (far back, at tile and block edges, on both sides of every window's and chunk's edge), memories that must hold for
hundreds of tokens, decays at their ends, convolutions across portions, layer norms of rows with a large mean, first tokens, long decoding, odd sizes, the
serving precision, graph replays, the engine's scheduler and the trace replay tool.

The error of a logits row is the root mean square of (got - want) with the mean taken off, over the row's own root mean square.  Rows computed with
exact_f32 differ from the float64 restatement by f32 rounding only: nine in ten rows stay within F32_TOL, every row within F32_WORST.  A wrong mechanism -
a lost state, a key one position off, a factor left out - moves rows by 1e-3 and more; the tests that aim at one show that first."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import rarutar_ref as R
import rarutar_synth as S

pytestmark = pytest.mark.gpu
F32_TOL = 2e-5
F32_WORST = 3e-4
BF16_TOL = 6e-2
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def row_errs(got, want):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean(-1))


def row_err(got, want):
    return float(row_errs(got, want).max())


def close(got, want):
    e = row_errs(got, want)
    return bool(e.max() <= F32_WORST and (len(e) < 10 or np.percentile(e, 90) <= F32_TOL))


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


class Rig:
    """A model folder, its weights for the oracle, and contexts of the product on it."""

    def __init__(self, pkg, folder, cfg, seed=0, tweak=None):
        self.cfg, self.W = cfg, S.weights(cfg, seed)
        if tweak:
            tweak(self.W)
        self.dir = S.write(folder, cfg, self.W)
        self.pkg = pkg
        self.model = pkg.Model(self.dir)

    def ctx(self, n_ctx=256, n_seq_max=4, exact=True, n_ubatch=64, graphs=True):
        return self.pkg.Context(self.model, n_ctx=n_ctx, n_batch=max(n_ctx, n_ubatch), n_ubatch=n_ubatch, n_seq_max=n_seq_max, exact_f32=exact, use_graphs=graphs)

    def ref(self, tokens, layers=False, without=()):
        taps = [] if layers else None
        out = R.forward(self.cfg, self.W, tokens, taps, without).numpy()
        return (out, np.stack([t.numpy() for t in taps])) if layers else out


def feed(ctx, tokens, start=0, seq=0, want_all=True):
    """One decode call for tokens[start:] of a sequence; returns the logits of every fed position."""
    n = len(tokens)
    assert ctx.decode(tokens, list(range(start, start + n)), seq=[seq] * n, logits=[1] * n if want_all else None) == 0
    return np.stack([ctx.logits(i) for i in range(n)]) if want_all else ctx.logits(-1)[None]


def feed_in_portions(ctx, tokens, sizes, seq=0, start=0):
    out, at, k = [], start, 0
    while at < len(tokens):
        n = min(sizes[k % len(sizes)], len(tokens) - at)
        out.append(feed(ctx, tokens[at:at + n], at, seq))
        at += n
        k += 1
    return np.concatenate(out)


def one_by_one(ctx, tokens, start=0, seq=0):
    return np.concatenate([feed(ctx, [tokens[i]], i, seq) for i in range(start, len(tokens))])


FULL = [S.parallel(mlp=S.dense()),
        S.attention(mlp=S.dense(20, 0.8)),
        S.mamba2(mlp=S.dense(56, 3.0)),
        S.parallel(heads=4, kv_heads=4, dim=8, vdim=16, size=5, dims=8, scaling=None, scale=0.5, left_scale=1.3, right_scale=0.4, r_heads=2, r_dim=20, r_vdim=8, tau=1.0, rank=16),
        S.attention(heads=4, kv_heads=1, dim=12, size=7, dims=12, scaling=S.yarn(2.0, 32), scale=0.5),
        S.mamba2(heads=4, vdim=16, state=8, groups=4, conv=1, norm_groups=1),
        S.mamba2(heads=3, vdim=8, state=20, groups=1, conv=5, norm_groups=2, mlp=S.dense())]


@pytest.fixture(scope="module")
def full(pkg, tmp_path_factory):
    """Every branch in one small model: scaled and plain rotation of whole heads and of parts, windows and chunks of several sizes, shared, own and one key head,
    tau 1 and 5, 1 - 5 taps, 1 - 4 groups and norm parts, layers without a feed-forward."""
    return Rig(pkg, tmp_path_factory.mktemp("rrt_full"), S.config(FULL), seed=3)


# ------------------------------------------------------------------------------------------ each mechanism alone
NOTHING = dict(heads=1, vdim=8, state=4, groups=1, conv=1, norm_groups=1)


@pytest.mark.parametrize("name,layers", [
    ("parallel", [S.parallel()]),
    ("parallel_plain_rotation", [S.parallel(scaling=None, dims=20)]),
    ("parallel_nothing_turns", [S.parallel(scaling=None, dims=0)]),
    ("parallel_window_one", [S.parallel(size=1)]),
    ("parallel_window_wider_than_the_prompt", [S.parallel(size=1000)]),
    ("parallel_every_head_its_own_key", [S.parallel(heads=3, kv_heads=3)]),
    ("parallel_one_key_head", [S.parallel(heads=5, kv_heads=1)]),
    ("parallel_wide_memory", [S.parallel(r_heads=2, r_dim=36, r_vdim=136)]),
    ("parallel_tau_one", [S.parallel(tau=1.0)]),
    ("attention", [S.attention()]),
    ("attention_scaled_rotation", [S.attention(scaling=S.yarn(8.0, 128, 16.0, 2.0), dims=20)]),
    ("attention_nothing_turns", [S.attention(dims=0)]),
    ("attention_chunks_of_one", [S.attention(size=1)]),
    ("attention_one_chunk", [S.attention(size=500)]),
    ("attention_one_key_head", [S.attention(heads=5, kv_heads=1)]),
    ("mamba2", [S.mamba2()]),
    ("mamba2_one_group", [S.mamba2(heads=5, groups=1, norm_groups=1)]),
    ("mamba2_every_head_its_own_group", [S.mamba2(heads=4, groups=4, norm_groups=8)]),
    ("mamba2_one_tap", [S.mamba2(conv=1)]),
    ("mamba2_two_taps", [S.mamba2(conv=2)]),
    ("mamba2_nine_taps", [S.mamba2(conv=9)]),
    ("mamba2_wide_heads", [S.mamba2(heads=2, vdim=72, state=40, groups=2, norm_groups=2)]),
    ("dense", [S.mamba2(mlp=S.dense(), **NOTHING)]),
    ("dense_tight_limit", [S.mamba2(mlp=S.dense(limit=0.1), **NOTHING)]),
    ("dense_wide_limit", [S.mamba2(mlp=S.dense(limit=50.0), **NOTHING)]),
])
def test_mechanism_alone_matches_the_restatement(pkg, tmp_path, name, layers):
    """A prompt of few rows (the kernels of single-token steps), one long enough for the batch kernels, and single tokens; the stream behind every layer."""
    rig = Rig(pkg, tmp_path / name, S.config(layers), seed=11)
    for n in (13, 53, 100):
        t = toks(n, rig.cfg["vocab"], 5)
        want, taps = rig.ref(t, layers=True)
        c = rig.ctx(n_ubatch=128)
        c.enable_taps(True)
        got = feed(c, t)
        for r in range(taps.shape[0]):
            assert np.abs(c.layer_out(r, len(t)) - taps[r]).max() <= 1e-4 * max(1.0, np.abs(taps[r]).max()), (name, r)
        assert close(got, want)
        assert close(one_by_one(rig.ctx(), t), want)


def test_the_restatement_tells_the_parts_apart(pkg, tmp_path):
    """Each part moves the logits of this model by far more than the tolerance: the product can only agree with the restatement if it has every one."""
    cfg = S.config([S.parallel(scale=0.5, mlp=S.dense(limit=0.7)), S.attention(scale=0.8, size=16, scaling=S.yarn()), S.mamba2(mlp=S.dense(limit=1.0))])
    rig = Rig(pkg, tmp_path / "parts", cfg, seed=12)
    t = toks(40, rig.cfg["vocab"], 6)
    want = rig.ref(t)
    for part in ("mean", "norm_bias", "left", "right", "scales", "rotation", "yarn", "mscale", "left_gate", "window", "qk_norm", "raw_values", "sink", "gate", "chunk", "state", "decay",
                 "tau", "right_norm", "right_gate", "conv", "conv_bias", "skip", "z_gate", "gate_behind", "one_part", "groups", "limit", "plus_one"):
        assert row_err(rig.ref(t, without=(part,)), want) > 1e-2, part
    assert close(feed(rig.ctx(), t), want)
    assert close(feed_in_portions(rig.ctx(), t, [7, 2, 1, 11]), want)


@pytest.mark.parametrize("width", [72, 50, 640, 1032])
@pytest.mark.parametrize("kind", ["mean", "outlier", "first_entries"])
def test_layer_norm_of_lopsided_rows(pkg, tmp_path, width, kind):
    """Rows whose mean is hundreds of times their spread; rows with one huge entry; rows whose first entries lie far from the others: few rows (the norm inside the
    products), batches, single tokens.  What the layers add to the stream is compared (the logits are made against the same lopsided table)."""
    def tweak(W):
        E = W["embed"].float() * 20.0
        if kind == "mean":
            E += 1500.0 * torch.sign(torch.randn(E.shape[0], 1, generator=torch.Generator().manual_seed(1)))
        elif kind == "outlier":
            E[:, 7] += 9000.0
        else:
            E[:, :max(width // 3, 8)] += 600.0
        W["embed"] = E.to(torch.bfloat16)
    rig = Rig(pkg, tmp_path / "ln", S.config([S.mamba2(mlp=S.dense(), **NOTHING), S.parallel(mlp=S.dense())], width=width, scale=1.0), seed=14, tweak=tweak)
    t = toks(40, 97, 15)
    x0 = rig.W["embed"].double()[t].numpy()
    _, taps = rig.ref(t, layers=True)

    def check(c, lo, hi):
        for r in range(2):
            got = c.layer_out(r, hi - lo).astype(np.float64) - x0[lo:hi]
            want = taps[r][lo:hi] - x0[lo:hi]
            rounding = np.abs(x0[lo:hi]).max() * 2.0 ** -24 * 4           # of the sums into the stream itself
            err = np.sqrt(((got - want) ** 2).mean(-1))
            assert (err <= 2e-4 * np.sqrt((want ** 2).mean(-1)) + rounding).all(), (r, lo, hi, err.max())

    for n in (1, 4, 16, 40):
        c = rig.ctx()
        c.enable_taps(True)
        feed(c, t[:n])
        check(c, 0, n)
    c = rig.ctx()
    c.enable_taps(True)
    for i in range(12):
        feed(c, [t[i]], i)
        check(c, i, i + 1)


def test_short_convolutions_reach_over_portions(pkg, tmp_path):
    """The oldest tap outweighs the others by far: a portion's first rows are made of what the sequence's slot remembers - portions shorter and longer than the
    taps, single tokens, two sequences in turn, and a new sequence in a slot whose predecessor left inputs behind."""
    def tweak(W):
        for il in (0, 1):
            W[f"l{il}.mix.conv"][:, 0] *= 6.0
    rig = Rig(pkg, tmp_path / "conv", S.config([S.mamba2(conv=6, mlp=S.dense()), S.mamba2(heads=2, vdim=16, state=16, groups=1, conv=4)]), seed=19, tweak=tweak)
    V = rig.cfg["vocab"]
    a, b = toks(60, V, 20), toks(47, V, 21)
    wa, wb = rig.ref(a), rig.ref(b)
    for sizes in ([1], [2], [3, 1, 4], [5, 6, 7], [20, 2, 40]):
        assert close(feed_in_portions(rig.ctx(), a, sizes), wa), sizes
    c = rig.ctx()
    got, at = [[], []], [0, 0]
    for na, nb in [(3, 20), (2, 2), (1, 1), (9, 1), (1, 7), (1, 1), (29, 1), (2, 10), (12, 4)]:
        tk = a[at[0]:at[0] + na] + b[at[1]:at[1] + nb]
        ps = list(range(at[0], at[0] + na)) + list(range(at[1], at[1] + nb))
        assert c.decode(tk, ps, seq=[0] * na + [1] * nb, logits=[1] * len(tk)) == 0
        rows = np.stack([c.logits(i) for i in range(len(tk))])
        got[0].append(rows[:na]); got[1].append(rows[na:])
        at[0] += na; at[1] += nb
    assert at == [60, 47] and close(np.concatenate(got[0]), wa) and close(np.concatenate(got[1]), wb)
    assert c.kv_seq_rm(0, -1, -1)
    assert close(feed_in_portions(c, b, [2, 1, 30], seq=0), wb)


# ------------------------------------------------------------------------------------------ prompts, single tokens, portions
def test_prompt_equals_token_by_token(full):
    t = toks(45, full.cfg["vocab"], 1)
    want = full.ref(t)
    whole = feed(full.ctx(), t)
    single = one_by_one(full.ctx(), t)
    assert close(whole, want) and close(single, want)
    assert close(single, whole)


@pytest.mark.parametrize("sizes", [[2], [3, 2, 7], [17, 2, 2, 30], [64, 5], [1, 2, 1, 9], [12, 11, 13], [31, 1, 32, 33], [1, 1, 2, 1, 3]])
def test_portions_of_any_size(full, sizes):
    """Portions that end on and beside the kernels' chunks (8, 16, 32 and 64 tokens), that cut a convolution's taps, and portions above 32 that the engine cuts
    again."""
    t = toks(97, full.cfg["vocab"], 2)
    got = feed_in_portions(full.ctx(n_ubatch=32), t, sizes)
    assert close(got, full.ref(t))


def test_long_decoding_after_a_prompt(full):
    t = toks(300, full.cfg["vocab"], 4)
    c = full.ctx(n_ctx=320)
    got = np.concatenate([feed(c, t[:40]), one_by_one(c, t, 40)])
    assert close(got, full.ref(t))


def test_the_first_tokens_of_a_sequence(full):
    """Position 0 sees one key, the memory is empty, the convolutions reach in front of the sequence."""
    t = toks(4, full.cfg["vocab"], 9)
    want = full.ref(t)
    assert close(feed(full.ctx(), t), want)
    assert close(one_by_one(full.ctx(), t), want)
    assert close(feed_in_portions(full.ctx(), t, [1, 3]), want)
    assert close(feed(full.ctx(), t[:1]), want[:1])


# ------------------------------------------------------------------------------------------ batches, cells and slots used again
def test_unequal_requests_in_one_batch_equal_each_alone(full):
    V = full.cfg["vocab"]
    reqs = [toks(n, V, 120 + i) for i, n in enumerate((37, 9, 61, 1))]
    want = [full.ref(r) for r in reqs]
    c = full.ctx(n_ctx=192, n_ubatch=48)                     # (48 cells per sequence region: the 61-token request spills into its neighbours')
    at = [0] * len(reqs)
    got = [[] for _ in reqs]
    plan = [(5, 1, 30, 1), (2, 1, 2, 0), (1, 1, 29, 0), (29, 6, 0, 0), (0, 0, 0, 0)]
    while any(at[i] < len(reqs[i]) for i in range(len(reqs))):
        for step in plan:
            tk, ps, sq, owner = [], [], [], []
            for i, n in enumerate(step):
                n = min(n if n else 1, len(reqs[i]) - at[i])
                tk += reqs[i][at[i]:at[i] + n]; ps += list(range(at[i], at[i] + n)); sq += [i] * n; owner += [i] * n
                at[i] += n
            if not tk:
                continue
            assert c.decode(tk, ps, seq=sq, logits=[1] * len(tk)) == 0
            for j, i in enumerate(owner):
                got[i].append(c.logits(j))
    for i in range(len(reqs)):
        assert close(np.stack(got[i]), want[i]), i


def test_a_sequence_that_comes_back_later_in_the_batch(full):
    """Rows of one sequence in two runs of the same batch, another sequence between them: the second run must start from the state the first one left."""
    V = full.cfg["vocab"]
    a, b = toks(20, V, 83), toks(6, V, 81)
    c = full.ctx()
    tk = a[:7] + b + a[7:20]
    ps = list(range(7)) + list(range(6)) + list(range(7, 20))
    sq = [0] * 7 + [1] * 6 + [0] * 13
    assert c.decode(tk, ps, seq=sq, logits=[1] * len(tk)) == 0
    got = np.stack([c.logits(i) for i in range(len(tk))])
    assert close(np.concatenate([got[:7], got[13:]]), full.ref(a))
    assert close(got[7:13], full.ref(b))


def test_cells_and_state_slots_are_used_again(full):
    """A context with room for one request at a time: every request takes the cells and the slot its predecessor gave back - a memory that kept anything
    of the predecessor would show at once; then two live requests, one ends and a third takes its slot beside the survivor."""
    V = full.cfg["vocab"]
    c = full.ctx(n_ctx=64, n_seq_max=2)
    for k in range(5):
        t = toks(50 + k, V, 40 + k)
        got = feed_in_portions(c, t, [13, 2, 21], seq=k % 2)
        assert close(got, full.ref(t)), k
        assert c.kv_used() == len(t)
        assert c.kv_seq_rm(k % 2, -1, -1)
        assert c.kv_used() == 0
    a, b, d = toks(30, V, 50), toks(34, V, 51), toks(28, V, 52)
    ga = feed(c, a, 0, 0)
    gb = feed(c, b[:20], 0, 1)
    assert c.kv_seq_rm(0, -1, -1)
    gd = feed(c, d, 0, 0)
    gb = np.concatenate([gb, feed(c, b[20:], 20, 1)])
    for got, t in ((ga, a), (gb, b), (gd, d)):
        assert close(got, full.ref(t))


def test_a_recurrent_sequence_cannot_be_cut_back_but_can_be_copied(full):
    t = toks(40, full.cfg["vocab"], 7)
    c = full.ctx()
    feed(c, t[:25])
    assert not c.kv_seq_rm(0, 12, -1)                           # the state has absorbed positions 12 .. 24
    c.kv_seq_cp(0, 2, 0, -1)                                    # cells and state of the whole sequence
    tail = toks(15, full.cfg["vocab"], 8)
    got0 = feed(c, t[25:], 25, 0)
    got2 = feed(c, tail, 25, 2)
    assert close(got0, full.ref(t)[25:])
    assert close(got2, full.ref(t[:25] + tail)[25:])


def test_attention_layers_alone_can_be_cut_back(pkg, tmp_path):
    """No recurrence anywhere: a sequence's tail can be removed and fed again."""
    rig = Rig(pkg, tmp_path / "cut", S.config([S.attention(mlp=S.dense()), S.attention(size=9)]), seed=27)
    t, tail = toks(40, rig.cfg["vocab"], 28), toks(20, rig.cfg["vocab"], 29)
    c = rig.ctx()
    feed(c, t)
    assert c.kv_seq_rm(0, 17, -1)
    assert close(feed(c, tail, 17), rig.ref(t[:17] + tail)[17:])


# ------------------------------------------------------------------------------------------ keys and memories made loud
D0 = 9                                                          # the loud coordinate (of the first head): one that does not turn


def _loud_rig(pkg, folder, layer, gain=5.0, seed=4):
    """One attention layer with a nearly one-hot softmax: a coordinate of the first query head and of its key that does not turn is made loud through the rows of
    the two projections; the recurrence beside a windowed attention is silenced, so that a row depends on what its attention sees alone."""
    left = layer["type"] == "parallel"
    def tweak(W):
        p = "l0.mix.left." if left else "l0.mix."
        W[p + "q"][D0] *= gain
        W[p + "k"][D0] *= gain
        if left:
            W["l0.mix.right.o"] *= 0.0
        else:
            W["l0.mix.sink"] *= 0.0
    return Rig(pkg, folder, S.config([layer], width=48, vocab=50), seed=seed, tweak=tweak)


def _loud_sequence(rig, n, p0, askers, seed=6):
    """n tokens whose keys are quiet in the loud coordinate, except ONE token at position p0 whose key is the loudest of the vocabulary; the rows in `askers`
    hold the quiet token whose query asks for it most."""
    F64, W, eps, lc = torch.float64, rig.W, rig.cfg["norm"]["eps"], rig.cfg["layers"][0]
    h = R.layer_norm(W["embed"].to(F64) * rig.cfg["embedding"]["scale"], W["l0.norm1"], W["l0.norm1.b"], eps)
    left = lc["type"] == "parallel"
    p, mx = ("l0.mix.left.", lc["mixer"]["left"]) if left else ("l0.mix.", lc["mixer"])
    D = mx["dim"]
    q, k = R.lin(h, W, p + "q")[:, :D], R.lin(h, W, p + "k")[:, :D]
    if not left:
        q, k = R.rms_unit(q, eps), R.rms_unit(k, eps)
    q, k = q[:, D0], k[:, D0]
    loud = int(torch.argmax(k))
    quiet = [int(i) for i in torch.argsort(k.abs()) if int(i) != loud][:30]
    asker = max(quiet, key=lambda i: float(q[i]))
    t = [quiet[int(i)] for i in torch.randint(0, len(quiet), (n,), generator=torch.Generator().manual_seed(seed))]
    t[p0] = loud
    for r in askers:
        t[r] = asker
    return t, quiet


def _loud_layer(kind, size):
    if kind == "window":
        return S.parallel(heads=4, kv_heads=2, dim=12, vdim=16, size=size, dims=8, scale=1.0)
    return S.attention(heads=4, kv_heads=2, dim=12, size=size, dims=8, scale=1.0)


def _all_ways(rig, t, want, cuts, n_ubatch=128):
    """The whole prompt at once, portions that open and close at the cuts, and single tokens from each cut on."""
    n_ctx = (len(t) + 63) // 64 * 64
    assert close(feed(rig.ctx(n_ctx=n_ctx, n_ubatch=512), t), want)
    for r in cuts:
        assert close(feed_in_portions(rig.ctx(n_ctx=n_ctx, n_ubatch=n_ubatch), t, [r, 2, 100]), want), r
        assert close(feed_in_portions(rig.ctx(n_ctx=n_ctx, n_ubatch=n_ubatch), t, [r + 1, 100]), want), r
        c = rig.ctx(n_ctx=n_ctx, n_ubatch=n_ubatch)
        lo = max(r - 2, 1)
        assert close(np.concatenate([feed_in_portions(c, t[:lo], [128, 3, 100]), one_by_one(c, t, lo)]), want), r


@pytest.mark.parametrize("kind", ["window", "chunk"])
@pytest.mark.parametrize("p0,far", [(0, 300), (15, 250), (31, 97), (63, 129), (64, 448)])
def test_a_far_key_among_hundreds(pkg, tmp_path, kind, p0, far):
    """One loud key hundreds of positions back, at the first cell and at the edges of the kernels' tiles and of a cell region: the asking row far behind depends
    on it (the restatement with another token in its place changes that row outright)."""
    rig = _loud_rig(pkg, tmp_path / "loud", _loud_layer(kind, far + 4 if kind == "window" else p0 + far + 4))
    r = p0 + far
    t, quiet = _loud_sequence(rig, r + 7, p0, [r, r + 3])
    want = rig.ref(t)
    other = list(t)
    other[p0] = quiet[0]
    e = row_errs(rig.ref(other), want)
    assert e[r] > 0.01 and e[r + 3] > 0.01, (e[r], e[r + 3])     # (of the logits row's own spread; the mixer's share of the stream bounds it)
    _all_ways(rig, t, want, [r])


@pytest.mark.parametrize("kind", ["window", "chunk"])
def test_the_causal_edge(pkg, tmp_path, kind):
    """The loud key at position p0: the asking row at p0 + 1 sees it, the one at p0 - 1 must not - also when both are rows of the same batch."""
    rig = _loud_rig(pkg, tmp_path / "edge", _loud_layer(kind, 100))
    for p0 in (1, 15, 16, 32, 40):
        t, quiet = _loud_sequence(rig, p0 + 12, p0, [p0 - 1, p0 + 1])
        want = rig.ref(t)
        other = list(t)
        other[p0] = quiet[0]
        e = row_errs(rig.ref(other), want)
        assert e[p0 + 1] > 0.02 and e[p0 - 1] == 0.0, p0
        assert close(feed(rig.ctx(), t), want)
        assert close(feed_in_portions(rig.ctx(), t, [p0, 2, 5]), want)        # the key opens a portion
        assert close(feed_in_portions(rig.ctx(), t, [p0 + 1, 2, 5]), want)    # ... and closes one
        c = rig.ctx()
        assert close(np.concatenate([feed(c, t[:max(p0 - 1, 1)]), one_by_one(c, t, max(p0 - 1, 1))]), want)


@pytest.mark.parametrize("size", [1, 2, 7, 16, 33, 64, 100])
@pytest.mark.parametrize("p0", [3, 64])
def test_the_windows_edge(pkg, tmp_path, size, p0):
    """The row `size - 1` positions behind the loud key is the last that sees it, the next one does not: in prompts, portions that start between the two, and
    decoded tokens."""
    rig = _loud_rig(pkg, tmp_path / "window", _loud_layer("window", size))
    last = p0 + size - 1
    t, quiet = _loud_sequence(rig, last + 9, p0, [r for r in (last, last + 1) if r != p0])
    want = rig.ref(t)
    other = list(t)
    other[p0] = quiet[0]
    e = row_errs(rig.ref(other), want)
    assert e[last] > 0.01 and e[last + 1] == 0.0, e[last]
    _all_ways(rig, t, want, [last, last + 1])


@pytest.mark.parametrize("size", [1, 3, 16, 30, 64, 70])
@pytest.mark.parametrize("first", [True, False])
def test_the_chunks_edge(pkg, tmp_path, size, first):
    """Chunks count from position 0 whatever the portions: the loud key at the first or the last position of the second chunk is seen by the chunk's last row and by
    none of the next chunk's, and a row of the chunk in front of it never sees it."""
    rig = _loud_rig(pkg, tmp_path / "chunk", _loud_layer("chunk", size))
    p0 = size if first else 2 * size - 1
    last = 2 * size - 1
    t, quiet = _loud_sequence(rig, last + 9, p0, [r for r in (size - 1, last, last + 1) if r != p0])
    want = rig.ref(t)
    other = list(t)
    other[p0] = quiet[0]
    e = row_errs(rig.ref(other), want)
    assert e[last] > 0.01 and e[last + 1] == 0.0 and (size == p0 + 1 or e[size - 1] == 0.0), e[last]
    _all_ways(rig, t, want, sorted({max(p0, 1), last, last + 1}))


@pytest.mark.parametrize("kind", ["window", "chunk"])
def test_a_loud_key_of_another_sequence_is_not_seen(pkg, tmp_path, kind):
    """Two sequences share the cells a tile walks; the loud key belongs to the other one."""
    rig = _loud_rig(pkg, tmp_path / "foreign", _loud_layer(kind, 200))
    a, quiet = _loud_sequence(rig, 70, 20, [40])
    b = [quiet[int(i)] for i in torch.randint(0, len(quiet), (66,), generator=torch.Generator().manual_seed(8))]
    b[45] = a[40]
    wa, wb = rig.ref(a), rig.ref(b)
    c = rig.ctx(n_ctx=192, n_seq_max=2, n_ubatch=256)
    tk, ps, sq = [], [], []
    for lo, hi in ((0, 25), (25, 50), (50, 70)):                 # both sequences' cells interleave
        for s, t in ((0, a), (1, b)):
            part = t[lo:min(hi, len(t))]
            tk += part; ps += list(range(lo, lo + len(part))); sq += [s] * len(part)
    assert c.decode(tk, ps, seq=sq, logits=[1] * len(tk)) == 0
    rows = np.stack([c.logits(i) for i in range(len(tk))])
    sq = np.array(sq)
    assert close(rows[sq == 0], wa) and close(rows[sq == 1], wb)
    more = [(0, a[40], 70), (1, a[40], 66)]                      # and in single-token steps side by side
    assert c.decode([m[1] for m in more], [m[2] for m in more], seq=[m[0] for m in more], logits=[1, 1]) == 0
    assert close(np.stack([c.logits(0)]), rig.ref(a + [a[40]])[-1:]) and close(np.stack([c.logits(1)]), rig.ref(b + [a[40]])[-1:])


def test_a_loud_sink(pkg, tmp_path):
    """A sink that takes nearly all of the weight in one head and none in another; rows that see one key and rows that see many."""
    def tweak(W):
        W["l0.mix.sink"] = torch.tensor([6.0, -40.0, 2.0, 0.0], dtype=torch.bfloat16)
    rig = Rig(pkg, tmp_path / "sink", S.config([S.attention(heads=4, kv_heads=2, dim=16, dims=8, size=20, scale=0.2)]), seed=16, tweak=tweak)
    t = toks(70, rig.cfg["vocab"], 17)
    want = rig.ref(t)
    assert row_errs(rig.ref(t, without=("sink",)), want).min() > 1e-3
    assert close(feed(rig.ctx(n_ubatch=128), t), want)
    assert close(one_by_one(rig.ctx(), t), want)


def test_requests_that_come_and_go_beside_a_long_one(pkg, tmp_path):
    """A long request decodes while short requests beside it start, end and hand their cells and slots on."""
    cfg = S.config([S.attention(mlp=S.dense()), S.mamba2(mlp=S.dense()), S.parallel()])
    rig = Rig(pkg, tmp_path / "beside", cfg, seed=8)
    V = cfg["vocab"]
    long_t = toks(150, V, 70)
    c = rig.ctx(n_ctx=256, n_seq_max=3, n_ubatch=32)
    got_long = [feed(c, long_t[:30], 0, 0)]
    at, k = 30, 0
    while at < len(long_t):
        short = toks(5 + 3 * (k % 4), V, 200 + k)
        slot = 1 + k % 2
        tk = [long_t[at]] + short
        ps = [at] + list(range(len(short)))
        sq = [0] + [slot] * len(short)
        assert c.decode(tk, ps, seq=sq, logits=[1] * len(tk)) == 0
        rows = np.stack([c.logits(i) for i in range(len(tk))])
        got_long.append(rows[:1])
        assert close(rows[1:], rig.ref(short)), k
        assert c.kv_seq_rm(slot, -1, -1)
        at += 1
        k += 1
    assert close(np.concatenate(got_long), rig.ref(long_t))


@pytest.mark.parametrize("layer", [
    S.parallel(r_heads=2, r_dim=24, r_vdim=16, tau=16.0), S.parallel(r_heads=3, r_dim=64, r_vdim=80, tau=16.0), S.parallel(r_heads=1, r_dim=130, r_vdim=260, tau=16.0),
    S.mamba2(heads=4, vdim=16, state=24, groups=2), S.mamba2(heads=2, vdim=72, state=136, groups=1, norm_groups=2)])
def test_a_memory_that_holds_hundreds_of_tokens(pkg, tmp_path, layer):
    """Decays nearly open: what token 60 wrote is still read 240 and more tokens later (the restatement with another token there differs at those rows) -
    through micro-batches, portions of two and single tokens."""
    def tweak(W):
        if layer["type"] == "parallel":
            W["l0.mix.left.o"] *= 0.0
            W["l0.mix.right.a2.b"] = torch.full_like(W["l0.mix.right.a2.b"], 4.0)
            W["l0.mix.right.a2"] *= 0.3
        else:
            W["l0.mix.A_log"] = torch.full_like(W["l0.mix.A_log"], -5.0)
            W["l0.mix.D"] *= 0.0
    rig = Rig(pkg, tmp_path / "hold", S.config([layer], width=48, vocab=50), seed=5, tweak=tweak)
    t = toks(330, 50, 17)
    want = rig.ref(t)
    other = list(t)
    other[60] = (t[60] + 1) % 50
    assert np.median(row_errs(rig.ref(other), want)[300:]) > 1e-3
    assert close(feed(rig.ctx(n_ctx=384, n_ubatch=512), t), want)
    assert close(feed_in_portions(rig.ctx(n_ctx=384, n_ubatch=48), t, [100, 2, 2, 150]), want)
    c = rig.ctx(n_ctx=384)
    assert close(np.concatenate([feed_in_portions(c, t[:290], [64]), one_by_one(c, t, 290)]), want)


@pytest.mark.parametrize("bias,spread,tau", [(-30.0, 1.0, 1.0), (40.0, 1.0, 16.0), (0.0, 30.0, 0.5), (-4.0, 8.0, 16.0), (-200.0, 60.0, 2.0)])
def test_channel_decays_at_their_ends(pkg, tmp_path, bias, spread, tau):
    """Decays that close at once, stay open, or swing over their whole range from token to token and from channel to channel."""
    def tweak(W):
        W["l0.mix.left.o"] *= 0.0
        W["l0.mix.right.a2"] *= spread
        W["l0.mix.right.a2.b"] = (W["l0.mix.right.a2.b"].float() - 1.0 + bias).to(torch.bfloat16)
    rig = Rig(pkg, tmp_path / "decay", S.config([S.parallel(r_heads=2, r_dim=40, r_vdim=24, tau=tau)], width=48, vocab=50), seed=6, tweak=tweak)
    t = toks(150, 50, 18)
    want = rig.ref(t)
    assert close(feed(rig.ctx(n_ubatch=256), t), want)
    assert close(feed_in_portions(rig.ctx(), t, [33, 2, 17, 1]), want)
    c = rig.ctx()
    assert close(np.concatenate([feed(c, t[:60]), one_by_one(c, t, 60)]), want)


@pytest.mark.parametrize("dt_bias,A_log,spread", [(4.0, 3.0, 1.0), (-20.0, 0.0, 1.0), (30.0, -6.0, 1.0), (-2.0, 1.0, 20.0), (0.0, 5.0, 6.0)])
def test_head_decays_and_step_sizes_at_their_ends(pkg, tmp_path, dt_bias, A_log, spread):
    """Steps that write hard and forget at once, hardly write, write hard and keep, or swing from token to token."""
    def tweak(W):
        W["l0.mix.in"][-4:] *= spread
        W["l0.mix.dt_bias"] = (W["l0.mix.dt_bias"].float() + 1.0 + dt_bias).to(torch.bfloat16)
        W["l0.mix.A_log"] = (W["l0.mix.A_log"].float() + A_log).to(torch.bfloat16)
    rig = Rig(pkg, tmp_path / "steps", S.config([S.mamba2(heads=4, vdim=20, state=24, groups=2)], width=48, vocab=50), seed=7, tweak=tweak)
    t = toks(150, 50, 18)
    want = rig.ref(t)
    assert close(feed(rig.ctx(n_ubatch=256), t), want)
    assert close(feed_in_portions(rig.ctx(), t, [33, 2, 17, 1]), want)
    c = rig.ctx()
    assert close(np.concatenate([feed(c, t[:60]), one_by_one(c, t, 60)]), want)


# ------------------------------------------------------------------------------------------ other sizes
@pytest.mark.parametrize("name,layers,width,vocab", [
    ("ones", [S.parallel(heads=1, kv_heads=1, dim=2, vdim=1, size=1, dims=2, r_heads=1, r_dim=1, r_vdim=1, rank=1, mlp=S.dense(1)), S.attention(heads=1, kv_heads=1, dim=1, size=1, dims=0),
              S.mamba2(heads=1, vdim=1, state=1, groups=1, conv=1, norm_groups=1)], 24, 11),
    ("left_dim_160_vdim_272", [S.parallel(heads=2, kv_heads=1, dim=160, vdim=272, size=70, dims=96, scale=0.1)], 64, 50),
    ("left_dim_320_vdim_136", [S.parallel(heads=2, kv_heads=2, dim=320, vdim=136, size=40, dims=320, scale=0.06)], 64, 50),
    ("left_unaligned", [S.parallel(heads=3, kv_heads=3, dim=10, vdim=7, size=11, dims=6)], 50, 53),
    ("right_dim_27_vdim_33", [S.parallel(r_heads=3, r_dim=27, r_vdim=33, rank=5)], 44, 50),
    ("right_dim_128_vdim_64", [S.parallel(r_heads=2, r_dim=128, r_vdim=64, rank=16)], 64, 50),
    ("right_dim_64_vdim_256", [S.parallel(r_heads=2, r_dim=64, r_vdim=256, rank=24)], 64, 50),
    ("right_dim_300_vdim_200", [S.parallel(r_heads=1, r_dim=300, r_vdim=200, rank=40)], 64, 50),
    ("right_vdim_320", [S.parallel(r_heads=2, r_dim=16, r_vdim=320, rank=8)], 64, 50),
    ("right_seven_heads", [S.parallel(r_heads=7, r_dim=8, r_vdim=16, rank=70)], 64, 50),
    ("attention_dim_256", [S.attention(heads=3, kv_heads=1, dim=256, size=50, dims=128, scale=0.05)], 64, 50),
    ("attention_dim_336", [S.attention(heads=2, kv_heads=1, dim=336, size=90, dims=64, scale=0.05)], 64, 50),
    ("attention_dim_13", [S.attention(heads=4, kv_heads=2, dim=13, size=31, dims=4)], 50, 53),
    ("attention_40_heads", [S.attention(heads=40, kv_heads=8, dim=16, size=48, dims=16, scale=0.3)], 72, 50),
    ("mamba2_state_128_vdim_64", [S.mamba2(heads=4, vdim=64, state=128, groups=2, conv=4, norm_groups=2)], 64, 50),
    ("mamba2_state_200_vdim_100", [S.mamba2(heads=2, vdim=100, state=200, groups=2, conv=4, norm_groups=2)], 64, 50),
    ("mamba2_state_7_vdim_5", [S.mamba2(heads=9, vdim=5, state=7, groups=3, conv=2, norm_groups=3)], 50, 53),
    ("mamba2_wide_parts", [S.mamba2(heads=36, vdim=64, state=8, groups=4, conv=4, norm_groups=1)], 64, 50),
    ("wide_feed_forward_width_50", [S.mamba2(mlp=S.dense(1300), **NOTHING)], 50, 50),
    ("aligned_everything", [S.parallel(heads=8, kv_heads=4, dim=32, vdim=48, size=48, dims=32, r_heads=2, r_dim=64, r_vdim=64, rank=16, mlp=S.dense(96)),
                            S.attention(heads=4, kv_heads=2, dim=32, size=64, dims=16, mlp=S.dense(64)), S.mamba2(heads=8, vdim=32, state=32, groups=2, conv=4, norm_groups=2, mlp=S.dense(128))], 128, 256),
])
def test_other_sizes(pkg, tmp_path, name, layers, width, vocab):
    rig = Rig(pkg, tmp_path / name, S.config(layers, width=width, vocab=vocab), seed=13)
    t = toks(150, vocab, 14)
    want = rig.ref(t)
    assert close(feed(rig.ctx(n_ubatch=256), t), want), name
    assert close(feed_in_portions(rig.ctx(), t, [33, 2, 1, 17]), want), name
    c = rig.ctx()
    assert close(np.concatenate([feed(c, t[:120]), one_by_one(c, t, 120)]), want), name


def test_many_sequences_in_one_step(pkg, tmp_path):
    """Twenty sequences decode side by side (more rows than the few-row kernels take), then a prompt portion joins nineteen single tokens."""
    rig = Rig(pkg, tmp_path / "many", S.config([S.parallel(mlp=S.dense()), S.mamba2(), S.attention()]), seed=15)
    V = rig.cfg["vocab"]
    seqs = [toks(9 + k % 5, V, 500 + k) for k in range(20)]
    want = [rig.ref(s) for s in seqs]
    c = rig.ctx(n_ctx=1280, n_seq_max=20, n_ubatch=64)
    got = [[] for _ in seqs]
    for i in range(5):
        assert c.decode([s[i] for s in seqs], [i] * 20, seq=list(range(20)), logits=[1] * 20) == 0
        for k in range(20):
            got[k].append(c.logits(k))
    tk, ps, sq = [], [], []
    for k, s in enumerate(seqs):
        n = len(s) - 5 if k == 7 else 1
        tk += s[5:5 + n]; ps += list(range(5, 5 + n)); sq += [k] * n
    assert c.decode(tk, ps, seq=sq, logits=[1] * len(tk)) == 0
    for j, k in enumerate(sq):
        got[k].append(c.logits(j))
    for k in range(20):
        assert close(np.stack(got[k]), want[k][:len(got[k])]), k


def _random_layer(rng):
    pick = lambda xs: xs[int(rng.integers(len(xs)))]
    mlp = pick([None, S.dense(pick([24, 64]), pick([0.5, 1.0, 4.0]))])
    kind = pick(["parallel", "attention", "mamba2"])
    dim = pick([16, 24, 32, 48])
    heads, share = pick([1, 2, 4, 8]), pick([1, 2, 4])
    kv = heads // share if heads % share == 0 else heads
    scaling = pick([None, S.yarn(), S.yarn(1.0), S.yarn(32.0, 4096, 32.0, 1.0)])
    if kind == "parallel":
        return S.parallel(heads=heads, kv_heads=kv, dim=dim, vdim=pick([8, 16, 40]), size=pick([1, 3, 40, 64, 100]), base=pick([1e4, 5e5]), dims=pick([8, 16]), scaling=scaling, scale=dim ** -0.5,
                          left_scale=pick([0.5, 1.0, 1.5]), right_scale=pick([0.25, 1.0]), r_heads=pick([1, 2, 5]), r_dim=pick([8, 16, 40, 72]), r_vdim=pick([16, 24, 72]), tau=pick([1.0, 4.0, 16.0]),
                          rank=pick([4, 16]), mlp=mlp)
    if kind == "attention":
        return S.attention(heads=heads, kv_heads=kv, dim=dim, size=pick([1, 5, 32, 64, 100]), base=pick([1e3, 1e6]), dims=pick([0, 8, 16]), scaling=scaling, scale=pick([0.1, 0.5]), mlp=mlp)
    groups = pick([g for g in (1, 2, 4) if heads % g == 0])
    return S.mamba2(heads=heads, vdim=pick([8, 16, 72]), state=pick([8, 16, 48]), groups=groups, conv=pick([1, 2, 4, 5]), norm_groups=pick([1, 2, 4]), mlp=mlp)


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
def test_random_configurations(pkg, tmp_path, seed):
    """Four to eight layers of any kind in any order with sizes drawn from lists; a 400-token request in portions of changing size and single tokens beside a
    short request that comes and goes."""
    rng = np.random.default_rng(seed)
    layers = [_random_layer(rng) for _ in range(int(rng.integers(4, 9)))]
    cfg = S.config(layers, width=int(rng.choice([64, 88, 128])), vocab=int(rng.choice([101, 256])), scale=float(rng.choice([0.5, 1.0, 4.0])))
    rig = Rig(pkg, tmp_path / f"random{seed}", cfg, seed=100 + seed)
    V = cfg["vocab"]
    long_t, short = toks(400, V, 7 + seed), toks(23, V, 9 + seed)
    want_long, want_short = rig.ref(long_t), rig.ref(short)
    c = rig.ctx(n_ctx=512, n_seq_max=2, n_ubatch=128)
    got_long, got_short, at, sat = [], [], 0, 0
    sizes = [150, 2, 1, 64, 1, 1, 37, 3, 1, 1, 1, 90, 1, 2]
    k = 0
    while at < len(long_t):
        n = min(sizes[k % len(sizes)], len(long_t) - at)
        m = min([5, 1, 1, 9, 2][k % 5], len(short) - sat)
        tk = long_t[at:at + n] + short[sat:sat + m]
        ps = list(range(at, at + n)) + list(range(sat, sat + m))
        sq = [0] * n + [1] * m
        assert c.decode(tk, ps, seq=sq, logits=[1] * len(tk)) == 0
        rows = np.stack([c.logits(i) for i in range(len(tk))])
        got_long.append(rows[:n])
        got_short.append(rows[n:])
        at += n
        sat += m
        if sat == len(short):                                   # the short request ends, gives its cells and slot back and starts over
            assert close(np.concatenate(got_short), want_short), (seed, k)
            assert c.kv_seq_rm(1, -1, -1)
            got_short, sat = [], 0
        k += 1
    assert close(np.concatenate(got_long), want_long), seed


# ------------------------------------------------------------------------------------------ precision, graphs
def test_serving_precision(full):
    """exact_f32 off: batches round their activations to bf16 for the matrix cores; positions, scores, softmax, norms, decays, the recurrences
    and the stream stay f32.  Single tokens keep f32 activations."""
    t = toks(96, full.cfg["vocab"], 30)
    want = full.ref(t)
    exact = feed(full.ctx(n_ubatch=128), t)
    bf = feed(full.ctx(exact=False, n_ubatch=128), t)
    e = row_errs(bf, want)
    assert np.median(e) <= 2e-2 and np.percentile(e, 90) <= BF16_TOL, (np.median(e), np.percentile(e, 90), e.max())
    assert row_err(bf, exact) > 1e-5                              # (activations were rounded to bf16: another kernel ran)
    single = one_by_one(full.ctx(exact=False), t)
    assert close(single, want)


def test_graph_replays_equal_eager_steps(full):
    t = toks(40, full.cfg["vocab"], 31)
    outs = []
    for graphs in (True, False):
        c = full.ctx(graphs=graphs)
        feed(c, t[:8], want_all=False)
        rows = []
        for i in range(8, len(t)):
            rows.append(feed(c, [t[i]], i, want_all=False)[0])
            if i % 7 == 0:
                c.synchronize()
        outs.append(np.stack(rows))
    assert np.array_equal(outs[0], outs[1])
    assert close(outs[0], full.ref(t)[8:])


# ------------------------------------------------------------------------------------------ the engine and the tools
def test_greedy_generation_through_the_engine(pkg, full):
    """loadmodel -> chat completion through the slot scheduler, two requests side by side; the text is decimal token ids."""
    V = full.cfg["vocab"]
    e = pkg.Engine()
    try:
        st, body = e.load_model(llama_model_path=full.dir, model="rrt", ctx_len=256, n_parallel=2, ngl=100, exact_f32=True, user_prompt="", ai_prompt="", system_prompt="")
        assert st["status_code"] == 200 and not st["has_error"], (st, body)
        prompts = [toks(11, V, 60), toks(23, V, 61)]
        n_new = 12

        def greedy(p):
            seq = list(p)
            for _ in range(n_new + 1):
                seq.append(int(np.argmax(full.ref(seq)[-1])))
            return seq[len(p):]

        import threading
        out = [None, None]

        def run(i):
            res = e.chat_completion(model="rrt", messages=[{"role": "user", "content": " ".join(map(str, prompts[i]))}], max_tokens=n_new, temperature=0.0,
                                    repeat_penalty=1.0, frequency_penalty=0.0, presence_penalty=0.0)
            out[i] = res[-1]

        th = [threading.Thread(target=run, args=(i,)) for i in range(2)]
        [x.start() for x in th]
        [x.join() for x in th]
        for i in range(2):
            st, body = out[i]
            assert st["status_code"] == 200 and not st["has_error"], (st, body)
            got = [int(x) for x in body["choices"][0]["message"]["content"].split()]
            want = greedy(prompts[i])
            assert len(got) >= n_new and got[:n_new] == want[:n_new], (got, want)
    finally:
        e.close()


def test_trace_tool_with_a_pool_that_is_always_full(pkg, tmp_path):
    """Up to four live requests of unequal lengths fed in portions of changing size beside single tokens of the others, in a pool that holds exactly what
    the live requests need (each rounded up to 64 cells): a finished request's cells and state slot go to the next one at once.  Every position of every
    request is asked for and compared with the restatement, in both precisions."""
    cfg = S.config([S.parallel(heads=4, kv_heads=2, dim=16, vdim=24, size=37, dims=16, r_heads=2, r_dim=24, r_vdim=16, tau=8.0, mlp=S.dense(48)),
                    S.attention(heads=6, kv_heads=3, dim=16, size=50, dims=8, mlp=S.dense(40)),
                    S.mamba2(heads=4, vdim=24, state=16, groups=2, conv=4, norm_groups=2, mlp=S.dense(32)),
                    S.mamba2(heads=2, vdim=32, state=24, groups=1, conv=3, norm_groups=1)], width=88, vocab=211)
    rig = Rig(pkg, tmp_path / "pool", cfg, seed=31)
    V = cfg["vocab"]
    rng = np.random.default_rng(5)
    lengths = [150, 64, 97, 1, 33, 128, 70, 191, 2, 65]
    reqs = {f"q{i}": toks(n, V, 300 + i) for i, n in enumerate(lengths)}
    waiting, live, at = list(reqs), [], {}
    steps, need = [], 0
    while waiting or live:
        while waiting and len(live) < 4:
            r = waiting.pop(0)
            live.append(r)
            at[r] = 0
        need = max(need, sum((len(reqs[r]) + 63) // 64 * 64 for r in live))
        entries, end = [], []
        for k, r in enumerate(live):
            if len(live) > 1 and rng.random() < 0.2:
                continue                                         # a request may sit a step out
            n = int(rng.choice([1, 1, 1, 2, 3, 5, 17, 40])) if at[r] > 0 or k != 1 else len(reqs[r])
            n = min(n, len(reqs[r]) - at[r])
            entries.append({"id": r, "tokens": reqs[r][at[r]:at[r] + n], "want": list(range(n))})
            at[r] += n
            if at[r] == len(reqs[r]):
                end.append(r)
        steps.append({"step": len(steps), "entries": entries, "end": end})
        live = [r for r in live if r not in end]
    want = {r: rig.ref(t) for r, t in reqs.items()}
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", rig.dir, "--dtype", dtype, "--out", str(out), "--max-tokens", str(need)],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
        assert p.returncode == 0, p.stderr[-2000:]
        got = {r: [] for r in reqs}
        for st in steps:
            if not any(e["want"] for e in st["entries"]):
                continue
            rows = np.fromfile(out / f"{st['step']}.f32", "<f4").reshape(-1, V)
            k = 0
            for e in st["entries"]:
                got[e["id"]].append(rows[k:k + len(e["want"])])
                k += len(e["want"])
            assert k == len(rows)
        errs = np.concatenate([row_errs(np.concatenate(got[r]), want[r]) for r in reqs])
        if dtype == "float32":
            assert errs.max() <= F32_WORST and np.percentile(errs, 90) <= F32_TOL, (errs.max(), np.percentile(errs, 90))
        else:
            assert np.median(errs) <= 2e-2 and np.percentile(errs, 90) <= BF16_TOL, (np.median(errs), np.percentile(errs, 90), errs.max())
