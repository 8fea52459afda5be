"""CPU: the package's synthetic Rarutar writer (what bench.py loads) against the tests' own writer and restatement - same tensor names and shapes for a
configuration, a header that the safetensors reader of the tests parses, weights the restatement runs on, and the bytes-per-token count; and the
restatement's own small parts against hand-worked values."""
import json
import math
import struct

import torch

import rarutar_ref as R
import rarutar_synth as S

F64 = torch.float64


def _header(path):
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        return json.loads(f.read(n)), 8 + n


def test_package_writer_agrees_with_the_tests_writer(pkg, tmp_path):
    rs = pkg.rarutar_synth
    size = rs.RarutarSize("tiny", 40, 61, 4, 2, 12, 6, 9, 3, 10, 6, 5, 6, 3, 8, 16, 4, 10, 7, 2, 30, conv=3, pattern=("Pd", "A", "Md"))
    cfg = rs.write_synthetic_rarutar(str(tmp_path / "m"), size, seed=5)
    assert json.load(open(tmp_path / "m" / "config.json")) == cfg
    head, base = _header(tmp_path / "m" / "model.safetensors")
    mine_cfg = json.loads(json.dumps(cfg))
    mine_cfg["layers"][0]["rank"] = 5
    mine = S.weights(mine_cfg, seed=1)
    assert set(head) == set(mine)
    for name, t in mine.items():
        assert head[name]["shape"] == list(t.shape) and head[name]["dtype"] == "BF16", name
    from safetensors.torch import load_file
    W = load_file(str(tmp_path / "m" / "model.safetensors"))
    out = R.forward(cfg, W, list(range(17)))
    assert out.shape == (17, 61) and bool(torch.isfinite(out).all())
    # bytes one token reads: projections, feed-forwards, head, a table row
    par = (4 * 12 + 2 * (12 + 6) + 4 + 2 * 3 * 10 + 2 * 3 * 6 + 5) * 40 + 3 * 10 * 5 + 40 * (4 * 6 + 3 * 6)
    att = (6 * 8 + 3 * 8 + 6) * 40 + 40 * 6 * 8
    ssd = (2 * 4 * 10 + 2 * 2 * 7 + 4) * 40 + 40 * 4 * 10
    assert rs.weight_bytes_per_token(cfg, 5) == 2 * (40 + 61 * 40 + par + att + ssd + 2 * 3 * 30 * 40)


def test_bench_sizes_are_loadable_configurations(pkg):
    rs = pkg.rarutar_synth
    for s in rs.SIZES.values():
        cfg = rs.config_of(s)
        assert s.heads % s.kv_heads == 0 and s.l_heads % s.l_kv_heads == 0 and s.m_heads % s.groups == 0
        names = [n for n, _ in rs.tensor_shapes(cfg, s.rank)]
        assert len(set(names)) == len(names)
        assert {lc["type"] for lc in cfg["layers"]} == {"parallel", "attention", "mamba2"}
        other = pkg.tuterax_synth.SIZES[s.name]
        assert (s.width, s.vocab, s.ff, s.heads, s.kv_heads, s.dim, len(s.pattern)) == (other.width, other.vocab, other.ff, other.heads, other.kv_heads, other.dim, len(other.pattern))


def test_windows_and_chunks_by_hand():
    assert R.seen_window(4, 2).tolist() == [[True, False, False, False], [True, True, False, False], [False, True, True, False], [False, False, True, True]]
    assert R.seen_chunk(4, 3).tolist() == [[True, False, False, False], [True, True, False, False], [True, True, True, False], [False, False, False, True]]


def test_rotation_by_hand():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 9.0]]] * 3, dtype=F64)
    y = R.turn(x, {"base": 100.0, "dims": 4})                    # frequencies 1 and 1/10; entry 0 with 2, entry 1 with 3; entry 4 stays
    assert torch.allclose(y[0], x[0])
    for p in (1, 2):
        for a, (lo, hi) in ((p * 1.0, (0, 2)), (p * 0.1, (1, 3))):
            u, v = float(x[0, 0, lo]), float(x[0, 0, hi])
            assert abs(float(y[p, 0, lo]) - (u * math.cos(a) - v * math.sin(a))) < 1e-12
            assert abs(float(y[p, 0, hi]) - (v * math.cos(a) + u * math.sin(a))) < 1e-12
        assert float(y[p, 0, 4]) == 9.0
    # scaled: 8 entries, base 10^4, frequencies 1, 0.1, 0.01, 0.001; an original context of 100 turns pair 0 15.9 times, pair 1 1.59 times, pair 2 0.159 times
    f, m = R.turn_table({"base": 10000.0, "dims": 8, "scaling": {"factor": 4.0, "original": 100, "fast": 2.0, "slow": 0.5}})
    lo = math.floor(8 * math.log(100 / (2 * math.pi * 2.0)) / (2 * math.log(10000.0)))      # 0.9 -> 0
    hi = math.ceil(8 * math.log(100 / (2 * math.pi * 0.5)) / (2 * math.log(10000.0)))       # 1.5 -> 2
    assert (lo, hi) == (0, 2)
    assert torch.allclose(f, torch.tensor([1.0, 0.1 * (0.5 + 0.5 / 4), 0.01 / 4, 0.001 / 4], dtype=F64))
    assert abs(m - (1.0 + 0.1 * math.log(4.0))) < 1e-12


def test_layer_norm_and_sink_by_hand():
    y = R.layer_norm(torch.tensor([[1.0, 3.0]], dtype=F64), torch.tensor([2.0, 1.0]), torch.tensor([0.5, 0.0]), 3.0)
    assert torch.allclose(y, torch.tensor([[-2.0 / 2 + 0.5, 1.0 / 2]], dtype=F64))
    s, v = torch.tensor([[math.log(2.0), 0.0]] * 2, dtype=F64), torch.tensor([[4.0], [8.0]], dtype=F64)
    o = R.softmax_sum(s, torch.tensor([[True, False], [True, True]]), v, torch.tensor(math.log(3.0), dtype=F64))
    assert torch.allclose(o, torch.tensor([[2 * 4 / 5.0], [(2 * 4 + 8) / 6.0]], dtype=F64))


def test_decay_scan_and_convolution_by_hand():
    q, k = torch.tensor([[1.0, 0.0], [1.0, 2.0]], dtype=F64).reshape(2, 1, 2), torch.tensor([[3.0, 1.0], [0.0, 1.0]], dtype=F64).reshape(2, 1, 2)
    v, a = torch.tensor([10.0, 1.0], dtype=F64).reshape(2, 1, 1), torch.tensor([[0.9, 0.9], [0.5, 0.1]], dtype=F64).reshape(2, 1, 2)
    o = R.decay_scan(q, k, v, a).reshape(2)
    assert torch.allclose(o, torch.tensor([30.0, 0.5 * 30.0 + 2 * (0.1 * 10.0 + 1.0)], dtype=F64))
    u = torch.tensor([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0]], dtype=F64)
    y = R.causal_conv(u, torch.tensor([[0.5, 0.0, 1.0], [1.0, 2.0, 3.0]]), torch.tensor([0.0, 1.0]))
    assert torch.allclose(y[:, 0], torch.tensor([1.0, 2.0, 3.5], dtype=F64)) and torch.allclose(y[:, 1], torch.tensor([31.0, 81.0, 141.0], dtype=F64))
