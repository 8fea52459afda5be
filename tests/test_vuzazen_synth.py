"""CPU: the package's synthetic Vuzazen writer (what bench.py loads) against the tests' own writer and restatement - same tensor names and shapes for a
configuration, a header that the safetensors reader of the tests parses, weights the restatement runs on, and the bytes-per-token count; and the
restatement's own small parts against hand-worked values."""
import json
import math
import struct

import torch

import vuzazen_ref as R
import vuzazen_synth as S

F64 = torch.float64


def _header(path):
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        return json.loads(f.read(n)), 8 + n


def test_package_writer_agrees_with_the_tests_writer(pkg, tmp_path):
    vs = pkg.vuzazen_synth
    size = vs.VuzazenSize("tiny", 40, 61, 3, 10, 6, 2, 8, 4, 12, 20, 16, 4, 2, 12, 8, 30, 5, 2, 14, conv=3, buckets=17, pattern=("Md", "Le", "A", "Me"))
    cfg = vs.write_synthetic_vuzazen(str(tmp_path / "m"), size, seed=5)
    assert json.load(open(tmp_path / "m" / "config.json")) == cfg
    head, base = _header(tmp_path / "m" / "model.safetensors")
    mine = S.weights(cfg, seed=1)
    assert set(head) == set(mine)
    for name, t in mine.items():
        assert head[name]["shape"] == list(t.shape) and head[name]["dtype"] == "BF16", name
    from safetensors.torch import load_file
    W = load_file(str(tmp_path / "m" / "model.safetensors"))
    out = R.forward(cfg, W, list(range(17)))
    assert out.shape == (17, 61) and bool(torch.isfinite(out).all())
    # bytes one token reads: projections, the chosen experts only, routers, head, two table rows
    ml = (2 * 3 * 10 + 2 * 3 * 6 + 2 * 3) * 40 + 40 * 3 * 6
    la = (16 + 20 + 4 + 2) * 40 + 2 * 12 * 16 + 2 * (8 + 12) * 20 + 40 * 2 * 12
    at = (4 * 12 + 2 * (12 + 8) + 4) * 40 + 40 * 4 * 8
    ex = 5 * 40 + 2 * 3 * 14 * 40
    assert vs.weight_bytes_per_token(cfg) == 2 * (2 * 40 + 61 * 40 + 2 * ml + la + at + 3 * 30 * 40 + 2 * ex)


def test_bench_sizes_are_loadable_configurations(pkg):
    vs = pkg.vuzazen_synth
    for s in vs.SIZES.values():
        cfg = vs.config_of(s)
        assert s.heads % s.kv_heads == 0 and s.top <= s.n_expert and s.l_rot % 2 == 0
        names = [n for n, _ in vs.tensor_shapes(cfg)]
        assert len(set(names)) == len(names)
        assert {lc["type"] for lc in cfg["layers"]} == {"mlstm", "latent_attention", "attention"}
        other = pkg.novorax_synth.SIZES[s.name]
        assert (s.width, s.vocab, s.m_heads, s.m_dim, s.m_vdim, s.l_heads, s.kv_rank, s.q_rank) == \
            (other.width, other.vocab, other.m_heads, other.m_dim, other.m_vdim, other.heads, other.kv_rank, other.q_rank)


def test_bigram_rows_by_hand():
    bg = {"buckets": 10, "mul_prev": 3, "mul_cur": 4}
    assert R.bigram_row(None, 7, bg) == 10
    assert R.bigram_row(0, 0, bg) == 0
    assert R.bigram_row(7, 5, bg) == (21 + 20) % 10
    assert R.bigram_row(5, 7, bg) == (15 + 28) % 10


def test_mlstm_by_hand():
    # one head, one dim, one value column: the gates chosen so that every step's maximum switches sides
    q, k, v = torch.tensor([1.0, 2.0, -1.0], dtype=F64), torch.tensor([0.5, -1.0, 3.0], dtype=F64), torch.tensor([2.0, 1.0, -1.0], dtype=F64)
    i, f = torch.tensor([-2.0, 1.0, 0.0], dtype=F64), torch.tensor([-0.5, -0.1, -3.0], dtype=F64)
    o = R.mlstm_scan(q.reshape(3, 1, 1), k.reshape(3, 1, 1), v.reshape(3, 1, 1), i.reshape(3, 1), f.reshape(3, 1)).reshape(3)
    # unstabilised: C = sum of e^(i) k v and N = sum of e^(i) k under the decays; o = q C / max(|q N|, 1) up to the 1e-6 (m = 0 start: e^-m is 1 unscaled)
    C = N = 0.0
    m = 0.0
    for t in range(3):
        C = math.exp(f[t]) * C + math.exp(i[t]) * float(k[t] * v[t])
        N = math.exp(f[t]) * N + math.exp(i[t]) * float(k[t])
        m = max(float(f[t]) + m, float(i[t]))
        want = float(q[t]) * C / (max(abs(float(q[t]) * N), 1.0) + 1e-6 * math.exp(m))
        assert abs(float(o[t]) - want) < 1e-12, t


def test_convolution_by_hand():
    u = torch.tensor([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0]], dtype=F64)
    w = torch.tensor([[0.5, 0.0, 1.0], [1.0, 2.0, 3.0]])
    y = R.causal_conv(u, w)
    assert torch.allclose(y[:, 0], torch.tensor([1.0, 2.0, 3.5], dtype=F64))
    assert torch.allclose(y[:, 1], torch.tensor([30.0, 80.0, 140.0], dtype=F64))


def test_router_and_turn_by_hand():
    ids, w = R.route(torch.tensor([[0.0, 2.0, -1.0, 2.0]], dtype=F64), 3)
    assert ids.tolist() == [[1, 3, 0]]
    s = 1 / (1 + math.exp(-2.0))
    assert torch.allclose(w, torch.tensor([[s, s, 0.5]], dtype=F64))
    x = torch.tensor([[1.0, 2.0, 3.0, 4.0]] * 3, dtype=F64)
    y = R.turn_halves(x, 100.0)                                  # frequencies 1 and 1/10; entry 0 with 2, entry 1 with 3
    assert torch.allclose(y[0], x[0])
    for p in (1, 2):
        for a, (lo, hi) in ((p * 1.0, (0, 2)), (p * 0.1, (1, 3))):
            u, v = float(x[0, lo]), float(x[0, hi])
            assert abs(float(y[p, lo]) - (u * math.cos(a) - v * math.sin(a))) < 1e-12
            assert abs(float(y[p, hi]) - (v * math.cos(a) + u * math.sin(a))) < 1e-12
