"""Writer of synthetic Vuzazen folders (config.json + model.safetensors) with seeded random bf16 weights, numpy only: what bench.py loads when no real
checkpoint is at hand (novorax_synth.py, fidepel_synth.py, tuterax_synth.py and dinilorn_synth.py are the same for the other folder designs).  The sizes
resemble the layers of real models of that width: mLSTM, latent attention and mixed-score attention in turns, dense and routed feed-forwards."""
from __future__ import annotations

import json
import os
import struct
from dataclasses import dataclass

import numpy as np

from .novorax_synth import _bf16


@dataclass
class VuzazenSize:
    """`pattern`: M = mlstm, L = latent attention, A = attention with mixed scores, each followed by d (dense), e (experts) or nothing."""
    name: str
    width: int
    vocab: int
    m_heads: int           # mlstm
    m_dim: int
    m_vdim: int
    l_heads: int           # latent attention
    l_dim: int
    l_rot: int
    l_vdim: int
    kv_rank: int
    q_rank: int
    heads: int             # attention
    kv_heads: int
    dim: int
    vdim: int
    ff: int
    n_expert: int
    top: int
    expert_ff: int
    conv: int = 4
    buckets: int = 32749
    pattern: tuple = ("Md", "Le", "Md", "Ae")


SIZES = {
    "w1024": VuzazenSize("w1024", 1024, 32000, 4, 128, 256, 8, 64, 32, 64, 256, 384, 16, 4, 64, 64, 1920, 8, 2, 704),
    "w2048": VuzazenSize("w2048", 2048, 32000, 8, 128, 256, 16, 128, 64, 128, 512, 768, 16, 4, 128, 128, 3776, 8, 2, 1408),
    "w4096": VuzazenSize("w4096", 4096, 32000, 16, 128, 256, 32, 128, 64, 128, 512, 1536, 32, 8, 128, 128, 7360, 8, 2, 2752),
}


def config_of(s: VuzazenSize) -> dict:
    layers = []
    for code in s.pattern:
        if code[0] == "M":
            lc = {"type": "mlstm", "mixer": {"dim": s.m_dim, "gate_cap": 15.0, "heads": s.m_heads, "vdim": s.m_vdim}}
        elif code[0] == "L":
            lc = {"type": "latent_attention", "mixer": {"dim": s.l_dim, "heads": s.l_heads, "kv_rank": s.kv_rank, "q_rank": s.q_rank, "rot": {"base": 500000.0, "dims": s.l_rot},
                                                        "rot_dim": s.l_rot, "scale": float((s.l_dim + s.l_rot) ** -0.5), "vdim": s.l_vdim}}
        else:
            lc = {"type": "attention", "mixer": {"conv": s.conv, "dim": s.dim, "heads": s.heads, "kv_heads": s.kv_heads, "scale": float(s.dim ** -0.5), "vdim": s.vdim}}
        lc["mlp"] = {"kind": "dense", "ff": s.ff} if code[1:] == "d" else \
            {"kind": "moe", "expert": {"ff": s.expert_ff}, "router": {"experts": s.n_expert, "top": s.top}} if code[1:] == "e" else None
        layers.append(lc)
    return {"architecture": "Vuzazen", "embedding": {"bigram": {"buckets": s.buckets, "mul_cur": 11, "mul_prev": 37}, "scale": float(s.width ** 0.5)}, "layers": layers,
            "norm": {"eps": 1e-6}, "vocab": s.vocab, "width": s.width}


def tensor_shapes(cfg: dict) -> list:
    """(name, shape) of every tensor the configuration asks for (all bf16)."""
    W, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, W)), ("bigram", (cfg["embedding"]["bigram"]["buckets"] + 1, W)), ("final.norm", (W,))]
    for il, lc in enumerate(cfg["layers"]):
        p, m = f"l{il}.", lc["mixer"]
        pm = p + "mix."
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        out.append((p + "norm1", (W,)))
        if lc["type"] == "mlstm":
            out += [(pm + "q", (H * D, W)), (pm + "k", (H * D, W)), (pm + "v", (H * VD, W)), (pm + "g", (H * VD, W)), (pm + "norm", (H * VD,)),
                    (pm + "i", (H, W)), (pm + "i.b", (H,)), (pm + "f", (H, W)), (pm + "f.b", (H,))]
        elif lc["type"] == "latent_attention":
            R, KR, QR = m["rot_dim"], m["kv_rank"], m["q_rank"]
            out += [(pm + "dq", (QR, W)), (pm + "dq.norm", (QR,)), (pm + "uq", (H * (D + R), QR)), (pm + "dkv", (KR + R, W)), (pm + "dkv.norm", (KR,)),
                    (pm + "uk", (H * D, KR)), (pm + "uv", (H * VD, KR)), (pm + "g", (H, W))]
        else:
            G, taps = m["kv_heads"], m["conv"]
            out += [(pm + "q", (H * D, W)), (pm + "k", (G * D, W)), (pm + "v", (G * VD, W)), (pm + "q.norm", (H * D,)), (pm + "k.norm", (G * D,)),
                    (pm + "q.conv", (H * D, taps)), (pm + "k.conv", (G * D, taps)), (pm + "v.conv", (G * VD, taps)), (pm + "talk", (H, H)), (pm + "g", (H, W))]
        out.append((pm + "o", (W, H * VD)))
        mlp = lc.get("mlp")
        if mlp:
            out.append((p + "norm2", (W,)))
            names = ["mlp."] if mlp["kind"] == "dense" else [f"mlp.e{e}." for e in range(mlp["router"]["experts"])]
            ff = mlp["ff"] if mlp["kind"] == "dense" else mlp["expert"]["ff"]
            for nm in names:
                out += [(p + nm + "gate", (ff, W)), (p + nm + "up", (ff, W)), (p + nm + "down", (W, ff))]
            if mlp["kind"] == "moe":
                out.append((p + "mlp.router", (mlp["router"]["experts"], W)))
    return out


def write_synthetic_vuzazen(folder: str, size, seed: int = 0) -> dict:
    """Writes the folder; returns the configuration.  Matrices are N(0, 1 / in) (talk: the identity plus N(0, 1 / heads)), the embedding N(0, 1 / width), the
    bigram table N(0, 0.25), plain norm weights N(1, 0.1), the other vectors N(0, 0.1), forget-gate biases 3."""
    s = SIZES[size] if isinstance(size, str) else size
    cfg = config_of(s)
    rng = np.random.default_rng(seed)
    os.makedirs(folder, exist_ok=True)
    shapes = tensor_shapes(cfg)
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
                gain, rows_left = np.float32(0.5 if name == "bigram" else shape[1] ** -0.5), shape[0]
                while rows_left > 0:                        # in slabs: a wide table would be gigabytes of floats at once
                    r = min(rows_left, 4096)
                    x = rng.standard_normal((r, shape[1]), dtype=np.float32) * gain
                    if name.endswith(".talk"):
                        x += np.eye(r, dtype=np.float32)
                    f.write(_bf16(x).astype("<u2").tobytes())
                    rows_left -= r
            else:
                mean = 3.0 if name.endswith("f.b") else 1.0 if name.endswith((".q.norm", ".k.norm", ".dq.norm", ".dkv.norm", "mix.norm")) else 0.0
                f.write(_bf16(rng.standard_normal(shape, dtype=np.float32) * np.float32(0.1) + np.float32(mean)).astype("<u2").tobytes())
    os.replace(tmp, os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    return cfg


def weight_bytes_per_token(cfg: dict) -> int:
    """Weight bytes one decoded token reads: every layer's projections, of the routed experts only the chosen ones, the routers, two table rows, the head."""
    W, V = cfg["width"], cfg["vocab"]
    total = 2 * (2 * W + V * W)
    for lc in cfg["layers"]:
        m = lc["mixer"]
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        if lc["type"] == "mlstm":
            n = (2 * H * D + 2 * H * VD + 2 * H) * W
        elif lc["type"] == "latent_attention":
            n = (m["q_rank"] + m["kv_rank"] + m["rot_dim"] + H) * W + H * (D + m["rot_dim"]) * m["q_rank"] + H * (D + VD) * m["kv_rank"]
        else:
            n = (H * D + m["kv_heads"] * (D + VD) + H) * W
        n += W * H * VD
        mlp = lc.get("mlp")
        if mlp:
            n += 3 * mlp["ff"] * W if mlp["kind"] == "dense" else (mlp["router"]["experts"] + 3 * mlp["router"]["top"] * mlp["expert"]["ff"]) * W
        total += 2 * n
    return total
