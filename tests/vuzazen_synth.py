"""Small Vuzazen models for tests: configurations of chosen sizes, random bf16 weights from a seed, written as a folder
(config.json + model.safetensors) the loader reads.  The sizes are deliberately odd ones - head counts, head sizes, expert
counts and widths that share no factor with the kernels' tile sizes."""
from __future__ import annotations

import json
import os

import torch


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def mlstm(heads=3, dim=20, vdim=12, gate_cap=7.0, mlp=None):
    return {"type": "mlstm", "mixer": {"dim": dim, "gate_cap": gate_cap, "heads": heads, "vdim": vdim}, "mlp": mlp}


def latent(heads=3, dim=12, rot_dim=8, vdim=20, kv_rank=28, q_rank=36, base=3000.0, scale=0.3, mlp=None):
    return {"type": "latent_attention", "mixer": {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank, "rot": {"base": base, "dims": rot_dim}, "rot_dim": rot_dim,
                                                  "scale": scale, "vdim": vdim}, "mlp": mlp}


def attention(heads=6, kv_heads=2, dim=16, vdim=20, conv=3, scale=0.35, mlp=None):
    return {"type": "attention", "mixer": {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "vdim": vdim}, "mlp": mlp}


def config(layers, width=72, vocab=97, eps=1e-5, scale=3.5, buckets=53, mul_prev=13, mul_cur=5):
    return {"architecture": "Vuzazen", "embedding": {"bigram": {"buckets": buckets, "mul_cur": mul_cur, "mul_prev": mul_prev}, "scale": scale}, "layers": layers,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}
    width, vocab = cfg["width"], cfg["vocab"]

    def mat(n, k, gain=1.0):
        return (torch.randn(n, k, generator=g) * gain / k ** 0.5).to(torch.bfloat16)

    def vec(n, std=0.1, mean=0.0):
        return (torch.randn(n, generator=g) * std + mean).to(torch.bfloat16)

    W["embed"] = (torch.randn(vocab, width, generator=g) * 0.3).to(torch.bfloat16)
    W["bigram"] = (torch.randn(cfg["embedding"]["bigram"]["buckets"] + 1, width, generator=g) * 0.5).to(torch.bfloat16)
    W["final.norm"] = vec(width, 0.2)
    for il, lc in enumerate(cfg["layers"]):
        p, m = f"l{il}.", lc["mixer"]
        pm = p + "mix."
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        W[p + "norm1"] = vec(width, 0.2)
        if lc["type"] == "mlstm":
            for nm, rows in (("q", H * D), ("k", H * D), ("v", H * VD), ("g", H * VD)):
                W[pm + nm] = mat(rows, width, 1.5)
            W[pm + "norm"] = vec(H * VD, 0.2, 1.0)
            for nm, mean in (("i", 0.0), ("f", 2.0)):
                W[pm + nm] = mat(H, width, 1.5)
                W[pm + nm + ".b"] = vec(H, 0.5, mean)
        elif lc["type"] == "latent_attention":
            R, KR, QR = m["rot_dim"], m["kv_rank"], m["q_rank"]
            W[pm + "dq"], W[pm + "dq.norm"] = mat(QR, width, 1.5), vec(QR, 0.2, 1.0)
            W[pm + "uq"] = mat(H * (D + R), QR, 1.5)
            W[pm + "dkv"], W[pm + "dkv.norm"] = mat(KR + R, width, 1.5), vec(KR, 0.2, 1.0)
            W[pm + "uk"], W[pm + "uv"] = mat(H * D, KR, 1.5), mat(H * VD, KR, 1.5)
            W[pm + "g"] = mat(H, width, 2.0)
        else:
            G, taps = m["kv_heads"], m["conv"]
            for nm, rows in (("q", H * D), ("k", G * D), ("v", G * VD)):
                W[pm + nm] = mat(rows, width, 1.5)
                W[pm + nm + ".conv"] = vec(rows * taps, 0.7).reshape(rows, taps)
            W[pm + "q.norm"], W[pm + "k.norm"] = vec(H * D, 0.2, 1.0), vec(G * D, 0.2, 1.0)
            W[pm + "talk"] = (torch.eye(H) * 0.8 + torch.randn(H, H, generator=g) / H ** 0.5).to(torch.bfloat16)
            W[pm + "g"] = mat(H, width, 2.0)
        W[pm + "o"] = mat(width, H * VD)
        mlp = lc.get("mlp")
        if mlp:
            W[p + "norm2"] = vec(width, 0.2)
            parts = [("mlp.", mlp["ff"])] if mlp["kind"] == "dense" else [(f"mlp.e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
            for nm, ff in parts:
                W[p + nm + "gate"] = mat(ff, width, 2.0)
                W[p + nm + "up"] = mat(ff, width, 2.0)
                W[p + nm + "down"] = mat(width, ff)
            if mlp["kind"] == "moe":
                W[p + "mlp.router"] = mat(mlp["router"]["experts"], width, 2.0)
    return W


def write(folder, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(folder, "model.safetensors"))
    return str(folder)
