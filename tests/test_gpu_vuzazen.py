"""Vuzazen on the GPU against the float64 restatement in tests/vuzazen_ref.py (which processes whole sequences, with no cache, no state and no
batching): every mechanism alone, prompts against token-by-token decoding, portions down to two tokens, mixed batches, cells and state slots that are
used again, keys made loud on purpose (far back, at tile and block edges, at the causal edge), a memory that must hold for hundreds of tokens, convolutions
and bigram rows across portions, first tokens, long decoding, odd sizes, the serving precision, graph replays, the engine's scheduler and the trace
replay tool.

The error of a logits row is the root mean square of (got - want) with the mean taken off, over the row's own root mean square.  Rows computed with
exact_f32 differ from the float64 restatement by f32 rounding only: nine in ten rows stay within F32_TOL, every row within F32_WORST.  A wrong mechanism -
a lost state, a key one position off, a head's score left out of the mix - moves rows by 1e-3 and more; the tests that aim at one show that first."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import vuzazen_ref as R
import vuzazen_synth as S

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


FULL = [S.mlstm(mlp=S.dense()),
        S.attention(mlp=S.moe(experts=8, top=3, ff=16)),
        S.latent(mlp=S.moe(experts=5, top=1)),
        S.mlstm(heads=2, dim=8, vdim=40, gate_cap=15.0, mlp=None),
        S.attention(heads=4, kv_heads=4, dim=12, vdim=12, conv=1, mlp=None),
        S.latent(heads=5, dim=8, rot_dim=0, vdim=8, kv_rank=20, q_rank=12, mlp=S.dense(16)),
        S.attention(heads=4, kv_heads=1, dim=32, vdim=16, conv=5, mlp=S.moe(experts=3, top=2))]


@pytest.fixture(scope="module")
def full(pkg, tmp_path_factory):
    """Every branch in one small model: the recurrence with two caps, mixed-score attention with shared, own and one key head and 1 - 5 taps, latent attention
    with and without a turning part, dense and routed feed-forwards with top 1 - 3, layers without a feed-forward."""
    return Rig(pkg, tmp_path_factory.mktemp("vzz_full"), S.config(FULL), seed=3)


# ------------------------------------------------------------------------------------------ each mechanism alone
@pytest.mark.parametrize("name,layers", [
    ("mlstm", [S.mlstm()]),
    ("mlstm_wide_values", [S.mlstm(heads=2, dim=24, vdim=136)]),
    ("mlstm_tight_cap", [S.mlstm(gate_cap=0.5)]),
    ("latent", [S.latent()]),
    ("latent_nothing_turns", [S.latent(rot_dim=0)]),
    ("latent_one_pair_turns", [S.latent(rot_dim=2, base=50.0)]),
    ("attention", [S.attention()]),
    ("attention_every_head_its_own_key", [S.attention(heads=3, kv_heads=3)]),
    ("attention_one_key_head", [S.attention(heads=5, kv_heads=1)]),
    ("attention_one_tap", [S.attention(conv=1)]),
    ("attention_two_taps", [S.attention(conv=2)]),
    ("attention_nine_taps", [S.attention(conv=9)]),
    ("dense", [S.mlstm(heads=1, dim=8, vdim=8, mlp=S.dense())]),
    ("experts_top_one", [S.mlstm(heads=1, dim=8, vdim=8, mlp=S.moe(experts=5, top=1))]),
    ("experts_top_two", [S.mlstm(heads=1, dim=8, vdim=8, mlp=S.moe())]),
    ("experts_all_taken", [S.mlstm(heads=1, dim=8, vdim=8, mlp=S.moe(experts=4, top=4))]),
])
def test_mechanism_alone_matches_the_restatement(pkg, tmp_path, name, layers):
    """A prompt of few rows (the kernels of single-token steps), one long enough for the batch kernels, and single tokens; the stream behind every layer."""
    rig = Rig(pkg, tmp_path / name, S.config(layers), seed=11)
    for n in (13, 53):
        t = toks(n, rig.cfg["vocab"], 5)
        want, taps = rig.ref(t, layers=True)
        c = rig.ctx()
        c.enable_taps(True)
        got = feed(c, t)
        for r in range(taps.shape[0]):
            assert np.abs(c.layer_out(r, len(t)) - taps[r]).max() <= 1e-4 * max(1.0, np.abs(taps[r]).max()), (name, r)
        assert close(got, want)
        assert close(one_by_one(rig.ctx(), t), want)


def test_the_restatement_tells_the_parts_apart(pkg, tmp_path):
    """Each part moves the logits of this model by far more than the tolerance: the product can only agree with the restatement if it has every one."""
    cfg = S.config([S.mlstm(gate_cap=1.5, mlp=S.moe(experts=8, top=2)), S.attention(scale=0.6), S.latent(scale=0.5, mlp=S.moe(top=1))])
    rig = Rig(pkg, tmp_path / "parts", cfg, seed=12)
    t = toks(40, rig.cfg["vocab"], 6)
    want = rig.ref(t)
    for part in ("bigram", "previous", "state", "cap", "gate", "rotation", "latent_norm", "conv", "talk", "talk_turned", "qk_norm", "v_norm", "weight", "weight_in"):
        assert row_err(rig.ref(t, without=(part,)), want) > 1e-2, part
    assert row_errs(rig.ref(t, without=("first_row",)), want)[0] > 1e-2
    assert close(feed(rig.ctx(), t), want)
    assert close(feed_in_portions(rig.ctx(), t, [7, 2, 1, 11]), want)


def test_scores_mixed_with_an_uneven_matrix(pkg, tmp_path):
    """A mixing matrix that only moves scores between heads (head 0 is scored by head 3, the others by sums and differences): few rows, batches, single tokens."""
    def tweak(W):
        W["l0.mix.talk"] = torch.tensor([[0, 0, 0, 1], [1, -1, 0, 0], [0.5, 0, 2, -0.25], [0, 3, 0, 0]], dtype=torch.bfloat16)
    rig = Rig(pkg, tmp_path / "mix", S.config([S.attention(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.5)]), seed=17, tweak=tweak)
    t = toks(90, rig.cfg["vocab"], 18)
    want = rig.ref(t)
    assert row_err(rig.ref(t, without=("talk_turned",)), want) > 1e-2
    for n in (6, 15, 16, 17, 90):
        assert close(feed(rig.ctx(n_ubatch=128), t[:n]), want[:n]), n
    assert close(one_by_one(rig.ctx(), t), want)


def test_short_convolutions_reach_over_portions(pkg, tmp_path):
    """The oldest tap outweighs the others by far: a portion's first rows are made of what the sequence's slot remembers - portions shorter and longer than the
    taps, single tokens, two sequences in turn, and a new sequence in a slot whose predecessor left inputs behind."""
    def tweak(W):
        for nm in "qkv":
            W[f"l0.mix.{nm}.conv"][:, 0] *= 6.0
    rig = Rig(pkg, tmp_path / "conv", S.config([S.attention(conv=6, mlp=S.dense()), S.attention(heads=2, kv_heads=2, conv=4)]), seed=19, tweak=tweak)
    V = rig.cfg["vocab"]
    a, b = toks(60, V, 20), toks(47, V, 21)
    wa, wb = rig.ref(a), rig.ref(b)
    for sizes in ([1], [2], [3, 1, 4], [5, 6, 7], [20, 2, 40]):
        assert close(feed_in_portions(rig.ctx(), a, sizes), wa), sizes
    c = rig.ctx()
    got, at = [[], []], [0, 0]
    for na, nb in [(3, 20), (2, 2), (1, 1), (9, 1), (1, 7), (30, 2), (2, 10), (12, 4)]:
        tk = a[at[0]:at[0] + na] + b[at[1]:at[1] + nb]
        ps = list(range(at[0], at[0] + na)) + list(range(at[1], at[1] + nb))
        assert c.decode(tk, ps, seq=[0] * na + [1] * nb, logits=[1] * len(tk)) == 0
        rows = np.stack([c.logits(i) for i in range(len(tk))])
        got[0].append(rows[:na]); got[1].append(rows[na:])
        at[0] += na; at[1] += nb
    assert at == [60, 47] and close(np.concatenate(got[0]), wa) and close(np.concatenate(got[1]), wb)
    assert c.kv_seq_rm(0, -1, -1)
    assert close(feed_in_portions(c, b, [2, 1, 30], seq=0), wb)


def test_bigram_rows_across_portions_and_sequences(pkg, tmp_path):
    """The bigram table outweighs the tokens' own rows: a lost or foreign previous token at a portion's first row, or an ordinary row instead of the last one
    at a sequence's first token, changes that row outright."""
    def tweak(W):
        W["bigram"] *= 8.0
    rig = Rig(pkg, tmp_path / "bigram", S.config([S.latent(), S.mlstm()], buckets=1009, mul_prev=100003, mul_cur=70001), seed=23, tweak=tweak)
    V = rig.cfg["vocab"]
    a, b = toks(30, V, 24), toks(30, V, 25)
    wa, wb = rig.ref(a), rig.ref(b)
    assert row_errs(rig.ref(a, without=("previous",)), wa)[1:].min() > 1e-2 and row_errs(rig.ref(a, without=("first_row",)), wa)[0] > 1e-2
    assert close(feed(rig.ctx(), a), wa)
    c = rig.ctx(n_seq_max=2)
    got, at = [[], []], [0, 0]
    for na, nb in [(1, 2), (2, 1), (5, 1), (1, 9), (21, 17)]:
        tk = a[at[0]:at[0] + na] + b[at[1]:at[1] + nb]
        ps = list(range(at[0], at[0] + na)) + list(range(at[1], at[1] + nb))
        assert c.decode(tk, ps, seq=[0] * na + [1] * nb, logits=[1] * len(tk)) == 0
        rows = np.stack([c.logits(i) for i in range(len(tk))])
        got[0].append(rows[:na]); got[1].append(rows[na:])
        at[0] += na; at[1] += nb
    assert close(np.concatenate(got[0]), wa) and close(np.concatenate(got[1]), wb)
    assert c.kv_seq_rm(1, -1, -1)
    assert close(one_by_one(c, a, seq=1), wa)                    # (a sequence starts over: its first token has no predecessor again)


def test_a_model_of_latent_layers_keeps_its_previous_token(pkg, tmp_path):
    """No recurrent layer and no convolution: the previous token alone forbids cutting a sequence back, and travels with a copy."""
    rig = Rig(pkg, tmp_path / "latent_only", S.config([S.latent(mlp=S.dense())]), seed=26)
    t = toks(20, rig.cfg["vocab"], 27)
    c = rig.ctx()
    feed(c, t[:12])
    assert not c.kv_seq_rm(0, 6, -1)
    c.kv_seq_cp(0, 1, 0, -1)
    assert close(feed(c, t[12:], 12, 1), rig.ref(t)[12:])


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
    """Position 0 sees one key, the memory is empty, the convolutions reach in front of the sequence, the bigram row is the last one."""
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


# ------------------------------------------------------------------------------------------ keys and memories made loud
D0 = 3                                                          # the loud coordinate (of the first head)


def _loud_rig(pkg, folder, layer, gain=5.0, seed=4):
    """One attention layer with a nearly one-hot softmax: coordinate D0 of the first query head and of its key (the unrotated part of a latent layer) is made
    loud through the rows of the two projections; the bigram table is silent and the convolutions pass their input, so that a token alone decides its key."""
    def tweak(W):
        W["bigram"] *= 0.0
        q, k = ("uq", "uk") if layer["type"] == "latent_attention" else ("q", "k")
        W["l0.mix." + q][D0] *= gain
        W["l0.mix." + k][D0] *= gain
        if layer["type"] == "attention":
            for nm in "qkv":
                W[f"l0.mix.{nm}.conv"][:] = 0.0
                W[f"l0.mix.{nm}.conv"][:, -1] = 1.0
    return Rig(pkg, folder, S.config([layer], width=48, vocab=50), seed=seed, tweak=tweak)


def _loud_sequence(rig, n, p0, askers, seed=6):
    """n tokens whose keys are quiet in the loud coordinate, except ONE token at position p0 whose key is the loudest of the vocabulary; the rows in `askers`
    hold the quiet token whose query asks for it most."""
    F64, W, eps, lc = torch.float64, rig.W, rig.cfg["norm"]["eps"], rig.cfg["layers"][0]
    h = R.norm(W["embed"].to(F64) * rig.cfg["embedding"]["scale"], W["l0.norm1"], eps)
    p = "l0.mix."
    if lc["type"] == "attention":
        k = (R.rms_unit(R.lin(h, W, p + "k"), eps) * W[p + "k.norm"].to(F64))[:, D0]
        q = (R.rms_unit(R.lin(h, W, p + "q"), eps) * W[p + "q.norm"].to(F64))[:, D0]
    else:
        KR = lc["mixer"]["kv_rank"]
        k = R.lin(R.rms_unit(R.lin(h, W, p + "dkv")[:, :KR], eps) * W[p + "dkv.norm"].to(F64), W, p + "uk")[:, D0]
        q = R.lin(R.rms_unit(R.lin(h, W, p + "dq"), eps) * W[p + "dq.norm"].to(F64), W, p + "uq")[:, D0]
    loud = int(torch.argmax(k))
    quiet = [int(i) for i in torch.argsort(k.abs()) if int(i) != loud][:30]
    asker = max(quiet, key=lambda i: float(q[i]))
    t = [quiet[int(i)] for i in torch.randint(0, len(quiet), (n,), generator=torch.Generator().manual_seed(seed))]
    t[p0] = loud
    for r in askers:
        t[r] = asker
    return t, quiet


LOUD = {"attention": S.attention(heads=4, kv_heads=2, dim=16, vdim=16, scale=1.2), "latent": S.latent(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=24, q_rank=24, scale=0.8, base=1e6)}


@pytest.mark.parametrize("kind", ["attention", "latent"])
@pytest.mark.parametrize("p0,far", [(0, 300), (15, 250), (31, 97), (63, 129), (64, 448)])
def test_a_far_key_among_hundreds(pkg, tmp_path, kind, p0, far):
    """One loud key hundreds of positions back, at the first cell and at the edges of the kernels' tiles and of a cell region: the asking row far behind depends
    on it (the restatement with another token in its place changes that row outright).  Whole prompts, portions cut by the micro-batch, single tokens, and a
    prompt that ends just before the asking row."""
    rig = _loud_rig(pkg, tmp_path / "loud", LOUD[kind])
    r = p0 + far
    n = r + 7
    t, quiet = _loud_sequence(rig, n, p0, [r, r + 3])
    want = rig.ref(t)
    other = list(t)
    other[p0] = quiet[0]
    e = row_errs(rig.ref(other), want)
    assert e[r] > 0.01 and e[r + 3] > 0.01, (e[r], e[r + 3])     # (of the logits row's own spread; the mixer's share of the stream bounds it)
    n_ctx = (n + 63) // 64 * 64
    assert close(feed(rig.ctx(n_ctx=n_ctx, n_ubatch=512), t), want)
    assert close(feed_in_portions(rig.ctx(n_ctx=n_ctx, n_ubatch=128), t, [r, 2, 100]), want)    # the asking row opens a two-token portion
    assert close(feed_in_portions(rig.ctx(n_ctx=n_ctx, n_ubatch=128), t, [r + 1, 100]), want)    # ... and closes a prompt portion
    c = rig.ctx(n_ctx=n_ctx, n_ubatch=128)
    got = np.concatenate([feed_in_portions(c, t[:r - 2], [128, 3, 100]), one_by_one(c, t, r - 2)])
    assert close(got, want)


@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_the_causal_edge(pkg, tmp_path, kind):
    """The loud key at position p0: the asking row at p0 + 1 sees it, the one at p0 - 1 must not - also when both are rows of the same batch."""
    rig = _loud_rig(pkg, tmp_path / "edge", LOUD[kind])
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


@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_a_loud_key_of_another_sequence_is_not_seen(pkg, tmp_path, kind):
    """Two sequences share the cells a tile walks; the loud key belongs to the other one."""
    rig = _loud_rig(pkg, tmp_path / "foreign", LOUD[kind])
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


def test_requests_that_come_and_go_beside_a_long_one(pkg, tmp_path):
    """A long request decodes while short requests beside it start, end and hand their cells and slots on."""
    cfg = S.config([S.attention(mlp=S.moe()), S.mlstm(mlp=S.dense()), S.latent(mlp=S.moe(top=1))])
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


@pytest.mark.parametrize("size", [dict(heads=2, dim=24, vdim=16), dict(heads=3, dim=64, vdim=80), dict(heads=1, dim=128, vdim=64)])
def test_a_memory_that_holds_hundreds_of_tokens(pkg, tmp_path, size):
    """Forget gates nearly open: what token 60 wrote is still read 240 and more tokens later (the restatement with another token there differs at those rows) -
    through micro-batches, portions of two and single tokens."""
    def tweak(W):
        H = size["heads"]
        W["bigram"] *= 0.0
        W["l0.mix.f"] *= 0.1
        W["l0.mix.f.b"] = torch.linspace(6.0, 8.0, H).to(torch.bfloat16)
        W["l0.mix.i"] *= 0.3
    rig = Rig(pkg, tmp_path / "hold", S.config([S.mlstm(gate_cap=12.0, **size)], width=48, vocab=50), seed=5, tweak=tweak)
    t = toks(330, 50, 17)
    want = rig.ref(t)
    other = list(t)
    other[60] = (t[60] + 1) % 50
    assert np.median(row_errs(rig.ref(other), want)[300:]) > 2e-3
    assert close(feed(rig.ctx(n_ctx=384, n_ubatch=512), t), want)
    assert close(feed_in_portions(rig.ctx(n_ctx=384, n_ubatch=48), t, [100, 2, 2, 150]), want)
    c = rig.ctx(n_ctx=384)
    assert close(np.concatenate([feed_in_portions(c, t[:290], [64]), one_by_one(c, t, 290)]), want)


@pytest.mark.parametrize("f_bias,i_bias,spread", [(-6.0, 0.0, 1.0), (0.0, 9.0, 3.0), (9.0, -9.0, 1.0), (-12.0, -12.0, 1.0), (2.0, 0.0, 8.0)])
def test_gates_at_their_ends(pkg, tmp_path, f_bias, i_bias, spread):
    """Gates that forget at once, write hard, hardly write, close both, or swing over their whole range from token to token: the running maximum follows the input
    gate, the forget gate, or jumps between them, and the denominator's floor takes over."""
    def tweak(W):
        for nm, b in (("i", i_bias), ("f", f_bias)):
            W["l0.mix." + nm] *= spread
            W[f"l0.mix.{nm}.b"] = (W[f"l0.mix.{nm}.b"].float() * 0.3 + b).to(torch.bfloat16)
    rig = Rig(pkg, tmp_path / "gates", S.config([S.mlstm(heads=3, dim=20, vdim=28, gate_cap=15.0)], width=48, vocab=50), seed=6, tweak=tweak)
    t = toks(150, 50, 18)
    want = rig.ref(t)
    assert close(feed(rig.ctx(n_ubatch=256), t), want)
    assert close(feed_in_portions(rig.ctx(), t, [33, 2, 17, 1]), want)
    c = rig.ctx()
    assert close(np.concatenate([feed(c, t[:60]), one_by_one(c, t, 60)]), want)


# ------------------------------------------------------------------------------------------ other sizes
@pytest.mark.parametrize("name,layers,width,vocab", [
    ("ones", [S.mlstm(heads=1, dim=1, vdim=1, mlp=S.moe(experts=1, top=1, ff=1)), S.attention(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, mlp=S.dense(1)),
              S.latent(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1)], 24, 11),
    ("mlstm_dim_144_vdim_200", [S.mlstm(heads=2, dim=144, vdim=200)], 64, 50),
    ("mlstm_dim_128_vdim_64", [S.mlstm(heads=2, dim=128, vdim=64)], 64, 50),
    ("mlstm_dim_64_vdim_128", [S.mlstm(heads=2, dim=64, vdim=128)], 64, 50),
    ("mlstm_dim_300", [S.mlstm(heads=1, dim=300, vdim=72)], 64, 50),
    ("mlstm_dim_40_unaligned", [S.mlstm(heads=5, dim=40, vdim=7)], 44, 50),
    ("mlstm_dim_27_unaligned", [S.mlstm(heads=3, dim=27, vdim=33)], 44, 50),
    ("attention_dim_160_vdim_272", [S.attention(heads=2, kv_heads=1, dim=160, vdim=272, scale=0.1)], 64, 50),
    ("attention_dim_320_vdim_136", [S.attention(heads=2, kv_heads=2, dim=320, vdim=136, scale=0.06)], 64, 50),
    ("attention_dim_48_vdim_256", [S.attention(heads=3, kv_heads=1, dim=48, vdim=256, scale=0.15)], 64, 50),
    ("attention_dim_128_vdim_128_twelve_heads", [S.attention(heads=12, kv_heads=3, dim=128, vdim=128, scale=0.1)], 64, 50),
    ("attention_unaligned_heads", [S.attention(heads=4, kv_heads=2, dim=10, vdim=14), S.attention(heads=3, kv_heads=3, dim=16, vdim=7)], 50, 53),
    ("attention_dim_24", [S.attention(heads=4, kv_heads=2, dim=24, vdim=16)], 48, 53),
    ("attention_24_heads", [S.attention(heads=24, kv_heads=3, dim=16, vdim=8, scale=0.3)], 72, 50),
    ("attention_40_heads", [S.attention(heads=40, kv_heads=8, dim=16, vdim=16, scale=0.3)], 72, 50),
    ("attention_70_heads", [S.attention(heads=70, kv_heads=7, dim=16, vdim=16, scale=0.3)], 72, 50),
    ("latent_kv_rank_200", [S.latent(heads=3, kv_rank=200, q_rank=44, rot_dim=16)], 64, 50),
    ("latent_kv_rank_512", [S.latent(heads=2, dim=32, kv_rank=512, q_rank=64, rot_dim=64, vdim=32, scale=0.1)], 64, 50),
    ("latent_unaligned", [S.latent(heads=3, dim=7, kv_rank=29, q_rank=15, rot_dim=6, vdim=9)], 50, 50),
    ("latent_20_heads", [S.latent(heads=20, dim=8, kv_rank=48, q_rank=32, rot_dim=8, vdim=8)], 64, 50),
    ("seventy_experts", [S.mlstm(heads=1, dim=8, vdim=8, mlp=S.moe(experts=70, top=3, ff=8))], 40, 50),
    ("wide_experts_width_50", [S.mlstm(heads=1, dim=8, vdim=8, mlp=S.moe(experts=3, top=2, ff=130))], 50, 50),
    ("aligned_everything", [S.attention(heads=8, kv_heads=4, dim=32, vdim=48, conv=4, mlp=S.moe(experts=8, top=1, ff=64)), S.latent(heads=4, dim=32, rot_dim=32, vdim=48, kv_rank=64, q_rank=48, mlp=S.dense(96)),
                            S.mlstm(heads=2, dim=64, vdim=64, mlp=S.moe(experts=4, top=2, ff=32))], 128, 256),
])
def test_other_sizes(pkg, tmp_path, name, layers, width, vocab):
    rig = Rig(pkg, tmp_path / name, S.config(layers, width=width, vocab=vocab), seed=13)
    t = toks(150, vocab, 14)
    want = rig.ref(t)
    assert close(feed(rig.ctx(n_ubatch=256), t), want), name
    assert close(feed_in_portions(rig.ctx(), t, [33, 2, 1, 17]), want), name
    c = rig.ctx()
    assert close(np.concatenate([feed(c, t[:120]), one_by_one(c, t, 120)]), want), name


def test_a_wide_vocabulary_with_few_rows(pkg, tmp_path):
    rig = Rig(pkg, tmp_path / "vocab", S.config([S.mlstm(heads=1, dim=8, vdim=8)], width=64, vocab=4099), seed=15)
    t = toks(9, 4099, 16)
    want = rig.ref(t)
    for n in (1, 2, 3, 4):
        assert close(feed(rig.ctx(), t[:n]), want[:n]), n


def _random_layer(rng):
    pick = lambda xs: xs[int(rng.integers(len(xs)))]
    mlp = pick([None, S.dense(pick([24, 64])), "moe", "moe"])
    if mlp == "moe":
        experts = pick([2, 5, 8, 16])
        mlp = S.moe(experts=experts, top=pick([t for t in (1, 1, 2, 3) if t <= experts]), ff=pick([8, 24, 48]))
    kind = pick(["mlstm", "latent", "attention"])
    if kind == "mlstm":
        return S.mlstm(heads=pick([1, 2, 5]), dim=pick([16, 48, 64]), vdim=pick([16, 48, 80]), gate_cap=pick([2.0, 15.0]), mlp=mlp)
    if kind == "latent":
        dim, rot = pick([16, 32, 40]), pick([8, 16, 32])
        return S.latent(heads=pick([1, 4, 6]), dim=dim, rot_dim=rot, vdim=pick([16, 32, 80]), kv_rank=pick([32, 64, 96]), q_rank=pick([24, 48]), base=pick([500.0, 1e6]),
                        scale=(dim + rot) ** -0.5, mlp=mlp)
    heads, share = pick([1, 2, 4, 8, 12]), pick([1, 2, 4])
    kv = heads // share if heads % share == 0 else heads
    dim = pick([16, 32, 48, 64])
    return S.attention(heads=heads, kv_heads=kv, dim=dim, vdim=pick([16, 32, 72]), conv=pick([1, 2, 4, 5]), scale=dim ** -0.5, mlp=mlp)


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6])
def test_random_configurations(pkg, tmp_path, seed):
    """Four to eight layers of any kind in any order with sizes drawn from lists; a 400-token request in portions of changing size and single tokens beside a
    short request that comes and goes."""
    rng = np.random.default_rng(seed)
    layers = [_random_layer(rng) for _ in range(int(rng.integers(4, 9)))]
    cfg = S.config(layers, width=int(rng.choice([64, 88, 128])), vocab=int(rng.choice([101, 256])), buckets=int(rng.choice([31, 1000])), scale=float(rng.choice([1.0, 4.0])))
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
    """exact_f32 off: batches round their activations to bf16 for the matrix cores; positions, scores, softmax, norms, the router's arithmetic, the recurrence
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
        st, body = e.load_model(llama_model_path=full.dir, model="vzz", ctx_len=256, n_parallel=2, ngl=100, exact_f32=True, user_prompt="", ai_prompt="", system_prompt="")
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
            res = e.chat_completion(model="vzz", messages=[{"role": "user", "content": " ".join(map(str, prompts[i]))}], max_tokens=n_new, temperature=0.0,
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
    cfg = S.config([S.mlstm(heads=4, dim=16, vdim=24, mlp=S.dense(48)),
                    S.attention(heads=6, kv_heads=3, dim=16, vdim=24, conv=4, mlp=S.moe(experts=4, top=1, ff=48)),
                    S.latent(heads=4, dim=24, rot_dim=12, vdim=16, kv_rank=40, q_rank=32, mlp=S.moe(experts=8, top=2, ff=32)),
                    S.mlstm(heads=2, dim=32, vdim=16)], width=88, vocab=211)
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
