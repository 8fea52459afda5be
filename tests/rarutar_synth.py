"""Small Rarutar models for tests: configurations of chosen sizes, random bf16 weights from a seed, written as a folder
(config.json + model.safetensors) the loader reads.  The sizes are deliberately odd ones - head counts, head sizes, ranks
and widths that share no factor with the kernels' tile sizes."""
from __future__ import annotations

import json
import os

import torch


def dense(ff=44, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def yarn(factor=4.0, original=64, fast=8.0, slow=1.0):
    return {"factor": factor, "fast": fast, "original": original, "slow": slow}


def _rot(base, dims, scaling):
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = scaling
    return rot


def parallel(heads=6, kv_heads=2, dim=20, vdim=12, size=13, base=700.0, dims=16, scaling="yarn", scale=0.35, left_scale=0.7, right_scale=1.2,
             r_heads=3, r_dim=12, r_vdim=28, tau=5.0, rank=9, mlp=None):
    """`rank` (the inner size of the decay's low-rank projection) is a tensor's shape, not a key of the configuration."""
    lc = {"type": "parallel", "mixer": {
        "left": {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": size}, "rot": _rot(base, dims, yarn() if scaling == "yarn" else scaling), "scale": scale, "vdim": vdim},
        "left_scale": left_scale, "right": {"dim": r_dim, "heads": r_heads, "tau": tau, "vdim": r_vdim}, "right_scale": right_scale}, "mlp": mlp}
    lc["rank"] = rank
    return lc


def attention(heads=6, kv_heads=3, dim=20, size=24, base=300.0, dims=12, scaling=None, scale=0.6, mlp=None):
    return {"type": "attention", "mixer": {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": size}, "rot": _rot(base, dims, scaling), "scale": scale, "vdim": dim}, "mlp": mlp}


def mamba2(heads=6, vdim=10, state=14, groups=3, conv=3, norm_groups=4, mlp=None):
    return {"type": "mamba2", "mixer": {"conv": conv, "groups": groups, "heads": heads, "norm_groups": norm_groups, "state": state, "vdim": vdim}, "mlp": mlp}


def config(layers, width=72, vocab=97, eps=1e-5, scale=2.5):
    """A parallel layer keeps its `rank` here for `weights`; `write` leaves it out of config.json."""
    return {"architecture": "Rarutar", "embedding": {"scale": scale}, "layers": [dict(lc) for lc in layers], "norm": {"eps": eps}, "vocab": vocab, "width": width}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}
    width, vocab = cfg["width"], cfg["vocab"]

    def mat(n, k, gain=1.0):
        return (torch.randn(n, k, generator=g) * gain / k ** 0.5).to(torch.bfloat16)

    def vec(n, std=0.1, mean=0.0):
        return (torch.randn(n, generator=g) * std + mean).to(torch.bfloat16)

    def norm(name):
        W[name], W[name + ".b"] = vec(width, 0.3, 1.0), vec(width, 0.2)

    W["embed"] = (torch.randn(vocab, width, generator=g) * 0.3 + 0.1).to(torch.bfloat16)
    norm("final.norm")
    for il, lc in enumerate(cfg["layers"]):
        p, m = f"l{il}.", lc["mixer"]
        pm = p + "mix."
        norm(p + "norm1")
        if lc["type"] == "parallel":
            a, b = m["left"], m["right"]
            for nm, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"]), ("g", a["heads"])):
                W[pm + "left." + nm] = mat(rows, width, 1.5)
            W[pm + "left.o"] = mat(width, a["heads"] * a["vdim"])
            H, D, VD, R = b["heads"], b["dim"], b["vdim"], lc["rank"]
            for nm, rows in (("q", H * D), ("k", H * D), ("v", H * VD), ("g", H * VD), ("a1", R)):
                W[pm + "right." + nm] = mat(rows, width, 1.5)
            W[pm + "right.a2"], W[pm + "right.a2.b"] = mat(H * D, R, 2.0), vec(H * D, 1.0, 1.0)
            W[pm + "right.norm"] = vec(VD, 0.3, 1.0)
            W[pm + "right.o"] = mat(width, H * VD)
        elif lc["type"] == "attention":
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            W[pm + "q"], W[pm + "k"], W[pm + "g"] = mat(H * D, width, 1.5), mat(G * D, width, 1.5), mat(H, width, 2.0)
            W[pm + "sink"] = vec(H, 1.0)
            W[pm + "o"] = mat(width, H * D)
        else:
            H, VD, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
            C = H * VD + 2 * G * N
            W[pm + "in"] = mat(2 * H * VD + 2 * G * N + H, width, 1.5)
            W[pm + "conv"], W[pm + "conv.b"] = vec(C * m["conv"], 0.7).reshape(C, m["conv"]), vec(C, 0.3)
            W[pm + "dt_bias"], W[pm + "A_log"], W[pm + "D"] = vec(H, 0.7, -1.0), vec(H, 0.7), vec(H, 0.5, 1.0)
            W[pm + "norm"] = vec(H * VD, 0.3, 1.0)
            W[pm + "o"] = mat(width, H * VD)
        if lc.get("mlp"):
            norm(p + "norm2")
            ff = lc["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = mat(ff, width, 2.0), mat(ff, width, 2.0), mat(width, ff)
    return W


def write(folder, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    cfg = dict(cfg, layers=[{k: v for k, v in lc.items() if k != "rank"} for lc in cfg["layers"]])
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(folder, "model.safetensors"))
    return str(folder)
