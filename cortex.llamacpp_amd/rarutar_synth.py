"""Writer of synthetic Rarutar folders (config.json + model.safetensors) with seeded random bf16 weights, numpy only: what bench.py loads when no real
checkpoint is at hand (novorax_synth.py and its siblings are the same for the other folder designs).  The sizes resemble the layers of real models of that
width: attention and gated linear attention side by side, attention in chunks and the state-space recurrence in turns, each with a dense feed-forward."""
from __future__ import annotations

import json
import os
import struct
from dataclasses import dataclass

import numpy as np

from .novorax_synth import _bf16


@dataclass
class RarutarSize:
    """`pattern`: P = two mixers side by side, A = attention in chunks, M = state-space recurrence, each followed by d (dense) or nothing."""
    name: str
    width: int
    vocab: int
    l_heads: int           # side by side, left: windowed attention
    l_kv_heads: int
    l_dim: int
    l_vdim: int
    window: int
    r_heads: int           # ... right: gated linear attention
    r_dim: int
    r_vdim: int
    rank: int
    heads: int             # attention in chunks
    kv_heads: int
    dim: int
    chunk: int
    m_heads: int           # state-space recurrence
    m_vdim: int
    state: int
    groups: int
    ff: int
    conv: int = 4
    pattern: tuple = ("Pd", "Ad", "Pd", "Md")


SIZES = {
    "w1024": RarutarSize("w1024", 1024, 32000, 8, 4, 64, 64, 1024, 4, 64, 128, 16, 16, 4, 64, 1024, 16, 64, 64, 2, 2816),
    "w2048": RarutarSize("w2048", 2048, 32000, 8, 4, 128, 128, 1024, 4, 128, 256, 16, 16, 4, 128, 1024, 32, 64, 128, 2, 5632),
    "w4096": RarutarSize("w4096", 4096, 32000, 16, 8, 128, 128, 1024, 8, 128, 256, 32, 32, 8, 128, 1024, 64, 64, 128, 4, 11008),
}


def config_of(s: RarutarSize) -> dict:
    layers = []
    for code in s.pattern:
        if code[0] == "P":
            lc = {"type": "parallel", "mixer": {
                "left": {"dim": s.l_dim, "heads": s.l_heads, "kv_heads": s.l_kv_heads, "mask": {"size": s.window},
                         "rot": {"base": 500000.0, "dims": s.l_dim, "scaling": {"factor": 4.0, "fast": 32.0, "original": 8192, "slow": 1.0}},
                         "scale": float(s.l_dim ** -0.5), "vdim": s.l_vdim},
                "left_scale": 1.0, "right": {"dim": s.r_dim, "heads": s.r_heads, "tau": 16.0, "vdim": s.r_vdim}, "right_scale": 1.0}}
        elif code[0] == "A":
            lc = {"type": "attention", "mixer": {"dim": s.dim, "heads": s.heads, "kv_heads": s.kv_heads, "mask": {"size": s.chunk}, "rot": {"base": 1000000.0, "dims": s.dim // 2},
                                                 "scale": float(s.dim ** -0.5), "vdim": s.dim}}
        else:
            lc = {"type": "mamba2", "mixer": {"conv": s.conv, "groups": s.groups, "heads": s.m_heads, "norm_groups": s.groups, "state": s.state, "vdim": s.m_vdim}}
        lc["mlp"] = {"kind": "dense", "ff": s.ff, "limit": 7.0} if code[1:] == "d" else None
        layers.append(lc)
    return {"architecture": "Rarutar", "embedding": {"scale": 1.0}, "layers": layers, "norm": {"eps": 1e-6}, "vocab": s.vocab, "width": s.width}


def tensor_shapes(cfg: dict, rank: int) -> list:
    """(name, shape) of every tensor the configuration asks for (all bf16); rank: inner size of the decays' low-rank projections."""
    W, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, W)), ("final.norm", (W,)), ("final.norm.b", (W,))]
    for il, lc in enumerate(cfg["layers"]):
        p, m = f"l{il}.", lc["mixer"]
        pm = p + "mix."
        out += [(p + "norm1", (W,)), (p + "norm1.b", (W,))]
        if lc["type"] == "parallel":
            a, b = m["left"], m["right"]
            H, G, D, VD = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            out += [(pm + "left.q", (H * D, W)), (pm + "left.k", (G * D, W)), (pm + "left.v", (G * VD, W)), (pm + "left.g", (H, W)), (pm + "left.o", (W, H * VD))]
            H, D, VD = b["heads"], b["dim"], b["vdim"]
            out += [(pm + "right.q", (H * D, W)), (pm + "right.k", (H * D, W)), (pm + "right.v", (H * VD, W)), (pm + "right.g", (H * VD, W)), (pm + "right.o", (W, H * VD)),
                    (pm + "right.norm", (VD,)), (pm + "right.a1", (rank, W)), (pm + "right.a2", (H * D, rank)), (pm + "right.a2.b", (H * D,))]
        elif lc["type"] == "attention":
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            out += [(pm + "q", (H * D, W)), (pm + "k", (G * D, W)), (pm + "sink", (H,)), (pm + "g", (H, W)), (pm + "o", (W, H * D))]
        else:
            H, VD, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
            C = H * VD + 2 * G * N
            out += [(pm + "in", (2 * H * VD + 2 * G * N + H, W)), (pm + "conv", (C, m["conv"])), (pm + "conv.b", (C,)), (pm + "dt_bias", (H,)), (pm + "A_log", (H,)), (pm + "D", (H,)),
                    (pm + "norm", (H * VD,)), (pm + "o", (W, H * VD))]
        if lc.get("mlp"):
            ff = lc["mlp"]["ff"]
            out += [(p + "norm2", (W,)), (p + "norm2.b", (W,)), (p + "mlp.gate", (ff, W)), (p + "mlp.up", (ff, W)), (p + "mlp.down", (W, ff))]
    return out


def write_synthetic_rarutar(folder: str, size, seed: int = 0) -> dict:
    """Writes the folder; returns the configuration.  Matrices are N(0, 1 / in), the convolution taps N(0, 1 / taps), norm weights N(1, 0.1), the other vectors N(0, 0.1),
    decay biases around 2, step-size biases around -2."""
    s = SIZES[size] if isinstance(size, str) else size
    cfg = config_of(s)
    rng = np.random.default_rng(seed)
    os.makedirs(folder, exist_ok=True)
    shapes = tensor_shapes(cfg, s.rank)
    head, off = {}, 0
    for name, shape in shapes:
        n = int(np.prod(shape, dtype=np.int64)) * 2
        head[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [off, off + n]}
        off += n
    hj = json.dumps(head, separators=(",", ":")).encode()
    hj += b" " * ((8 - len(hj) % 8) % 8)
    tmp = os.path.join(folder, "model.safetensors.tmp")
    with open(tmp, "wb") as f:
        f.write(struct.pack("<Q", len(hj)))
        f.write(hj)
        for name, shape in shapes:
            if len(shape) == 2:
                gain, rows_left = np.float32(shape[1] ** -0.5), shape[0]
                while rows_left > 0:                        # in slabs: a wide table would be gigabytes of floats at once
                    r = min(rows_left, 4096)
                    f.write(_bf16(rng.standard_normal((r, shape[1]), dtype=np.float32) * gain).astype("<u2").tobytes())
                    rows_left -= r
            else:
                mean = 2.0 if name.endswith("a2.b") else -2.0 if name.endswith("dt_bias") else 1.0 if name.endswith(("norm", "norm1", "norm2", ".D")) else 0.0
                f.write(_bf16(rng.standard_normal(shape, dtype=np.float32) * np.float32(0.1) + np.float32(mean)).astype("<u2").tobytes())
    os.replace(tmp, os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    return cfg


def weight_bytes_per_token(cfg: dict, rank: int) -> int:
    """Weight bytes one decoded token reads: every layer's projections, a table row, the head."""
    W, V = cfg["width"], cfg["vocab"]
    total = 2 * (W + V * W)
    for lc in cfg["layers"]:
        m = lc["mixer"]
        if lc["type"] == "parallel":
            a, b = m["left"], m["right"]
            n = (a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"]) + a["heads"] + 2 * b["heads"] * (b["dim"] + b["vdim"]) + rank) * W
            n += b["heads"] * b["dim"] * rank + W * (a["heads"] * a["vdim"] + b["heads"] * b["vdim"])
        elif lc["type"] == "attention":
            n = (m["heads"] * (m["dim"] + 1) + m["kv_heads"] * m["dim"]) * W + W * m["heads"] * m["dim"]
        else:
            n = (2 * m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"] + m["heads"]) * W + W * m["heads"] * m["vdim"]
        if lc.get("mlp"):
            n += 3 * lc["mlp"]["ff"] * W
        total += 2 * n
    return total
