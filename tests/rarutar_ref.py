"""Plain, slow restatement of the Rarutar design in float64 torch, one function per mechanism.

Test infrastructure only: it shares no code with the product path (cortex.llamacpp_amd/), runs on the CPU and
processes whole sequences at once - no cache, no batching, the recurrences token by token.  Weights are a dict
name -> tensor, the configuration is the dict a model's config.json holds.

Notation: x [T, width] the residual stream of one sequence, positions 0 .. T-1; ln(y) = (y - mean) / sqrt(var + eps) * w + b;
u(y) = y / rms(y).
  embedding:  x_t = scale * E[t]
  layer:      x <- x + mixer(ln1(x));  x <- x + ff(ln2(x))   (a layer may have no ff)
  parallel:   left_scale * windowed attention + right_scale * gated linear attention, both on the same input
    left:     q, k, v of H / G / G heads; entry i < dims/2 of q and k pairs with entry i + dims/2 and turns by p * f_i (blended
              frequencies, cos and sin times a constant when the rotation is scaled);  s(i, j) = q_i.k_j scale for 0 <= i - j < size;
              softmax;  times sigmoid(Wg h)[head];  Wo
    right:    q = Wq h / sqrt(dim), k, v per head;  a = sigmoid(Wa2 Wa1 h + ba2)^(1/tau) per key channel;
              S <- a[:, None] S + k v^T;  o = S^T q;  u(o) w;  times silu(Wg h);  Wo
  attention:  v = k as projected; q and k turn, then u(q), u(k) per head;  j <= i and i // size == j // size;  softmax with one more
              term exp(sink_h) in the denominator;  times sigmoid(Wg h)[head];  Wo
  mamba2:     [z | x | B | C | dt] = Win h;  x, B, C through a causal convolution with bias and silu;  dt <- softplus(dt + dt_bias);
              S <- exp(-exp(A_log) dt) S + dt B x^T;  y = S^T C + D x;  y * silu(z), u over equal parts, times w;  Wo
  ff:         g = min(Wgate h, limit), u = clamp(Wup h, +-limit);  Wdown (g sigmoid(1.702 g) (u + 1))
  output:     logits = E ln_final(x)
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_unit(x, eps):
    """x over its root mean square along the last axis, eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps, without=()):
    """`without`: "mean" (nothing is taken off), "norm_bias"."""
    if "mean" not in without:
        x = x - x.mean(-1, keepdim=True)
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)
    return y if "norm_bias" in without else y + b.to(F64)


def lin(x, W, name):
    return x @ W[name].to(F64).T


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


# ---------------------------------------------------------------------------------------------- rotation
def turn_table(rot, without=()):
    """(radians per position of every pair, factor of cos and sin).  `without`: "yarn" (plain frequencies, factor 1), "mscale" (factor 1)."""
    n, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if not sc or "yarn" in without:
        return torch.tensor(f, dtype=F64), 1.0
    at = lambda turns: n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(at(sc["fast"])), 0), min(math.ceil(at(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1 - r))
    return torch.tensor(out, dtype=F64), 1.0 if "mscale" in without else 0.1 * math.log(sc["factor"]) + 1.0


def turn(x, rot, without=()):
    """x [T, heads, D] of positions 0 .. T-1: the first rot.dims entries of every head turn in pairs (i, i + dims/2)."""
    if not rot or rot["dims"] == 0 or "rotation" in without:
        return x
    n = rot["dims"]
    freq, mult = turn_table(rot, without)
    ang = torch.arange(x.shape[0], dtype=F64)[:, None, None] * freq
    c, s = torch.cos(ang) * mult, torch.sin(ang) * mult
    a, b = x[..., :n // 2], x[..., n // 2:n]
    return torch.cat([a * c - b * s, b * c + a * s, x[..., n:]], dim=-1)


# ---------------------------------------------------------------------------------------------- attention
def seen_window(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (i - j >= 0) & (i - j < size)


def seen_chunk(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def softmax_sum(s, seen, v, sink=None):
    """s [T, T] scores, seen [T, T]; sink: one more term in every row's denominator."""
    s = s.masked_fill(~seen, float("-inf"))
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.clamp(m, min=float(sink))
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink.to(F64) - m)
    return (e / den) @ v


def left_mixer(h, W, p, mx, eps, without=()):
    """`without`: "rotation", "yarn", "mscale", "left_gate", "window" (every earlier position is seen)."""
    T = h.shape[0]
    H, G, D, VD = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = turn(lin(h, W, p + "q").reshape(T, H, D), mx.get("rot"), without)
    k = turn(lin(h, W, p + "k").reshape(T, G, D), mx.get("rot"), without)
    v = lin(h, W, p + "v").reshape(T, G, VD)
    g = torch.sigmoid(lin(h, W, p + "g"))
    seen = seen_window(T, T if "window" in without else mx["mask"]["size"])
    heads = []
    for a in range(H):
        o = softmax_sum((q[:, a] @ k[:, a // (H // G)].T) * float(mx["scale"]), seen, v[:, a // (H // G)])
        heads.append(o if "left_gate" in without else o * g[:, a:a + 1])
    return lin(torch.cat(heads, -1), W, p + "o")


def attention(h, W, p, mx, eps, without=()):
    """`without`: "rotation", "qk_norm", "norm_first" (the unit norm in front of the rotation - the same thing unless cos and sin carry a factor), "sink", "gate",
    "chunk" (every earlier position is seen), "raw_values" (the values are the finished keys)."""
    T = h.shape[0]
    H, G, D = mx["heads"], mx["kv_heads"], mx["dim"]
    q = lin(h, W, p + "q").reshape(T, H, D)
    k = lin(h, W, p + "k").reshape(T, G, D)
    v = k
    unit = (lambda y: y) if "qk_norm" in without else (lambda y: rms_unit(y, eps))
    q, k = unit(turn(q, mx.get("rot"), without)), unit(turn(k, mx.get("rot"), without))
    if "raw_values" in without:
        v = k
    g = torch.sigmoid(lin(h, W, p + "g"))
    seen = seen_chunk(T, T if "chunk" in without else mx["mask"]["size"])
    heads = []
    for a in range(H):
        sink = None if "sink" in without else W[p + "sink"][a].to(F64)
        o = softmax_sum((q[:, a] @ k[:, a // (H // G)].T) * float(mx["scale"]), seen, v[:, a // (H // G)], sink)
        heads.append(o if "gate" in without else o * g[:, a:a + 1])
    return lin(torch.cat(heads, -1), W, p + "o")


# ---------------------------------------------------------------------------------------------- gated linear attention
def decay_scan(q, k, v, a):
    """q, k [T, H, D], v [T, H, VD], a [T, H, D] the decay of every row of the state -> o [T, H, VD]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    out = []
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def right_mixer(h, W, p, mx, eps, without=()):
    """`without`: "state" (every token sees only itself), "decay" (nothing fades), "tau" (tau = 1), "right_norm", "right_gate"."""
    T = h.shape[0]
    H, D, VD = mx["heads"], mx["dim"], mx["vdim"]
    q = lin(h, W, p + "q").reshape(T, H, D) * D ** -0.5
    k = lin(h, W, p + "k").reshape(T, H, D)
    v = lin(h, W, p + "v").reshape(T, H, VD)
    z = (lin(lin(h, W, p + "a1"), W, p + "a2") + W[p + "a2.b"].to(F64)).reshape(T, H, D)
    a = torch.exp(-softplus(-z) / (1.0 if "tau" in without else float(mx["tau"])))
    if "state" in without:
        a = torch.zeros_like(a)
    if "decay" in without:
        a = torch.ones_like(a)
    o = decay_scan(q, k, v, a)
    if "right_norm" not in without:
        o = rms_unit(o, eps)
    o = (o * W[p + "norm"].to(F64)).reshape(T, H * VD)
    if "right_gate" not in without:
        o = o * silu(lin(h, W, p + "g"))
    return lin(o, W, p + "o")


def parallel(h, W, p, mx, eps, without=()):
    """`without`: "left", "right", "scales"."""
    ls, rs = (1.0, 1.0) if "scales" in without else (float(mx["left_scale"]), float(mx["right_scale"]))
    out = torch.zeros_like(h)
    if "left" not in without:
        out = out + ls * left_mixer(h, W, p + "left.", mx["left"], eps, without)
    if "right" not in without:
        out = out + rs * right_mixer(h, W, p + "right.", mx["right"], eps, without)
    return out


# ---------------------------------------------------------------------------------------------- mamba2
def causal_conv(u, w, b):
    """u [T, C], w [C, taps], b [C]: the last tap meets the token itself, the ones before it the tokens before; zeros in front of the sequence."""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    return sum(pad[j:j + T] * w[:, j].to(F64) for j in range(taps)) + b.to(F64)


def mamba2(h, W, p, mx, eps, without=()):
    """`without`: "conv", "conv_bias", "state", "skip" (no D x), "z_gate", "gate_behind" (the gate multiplies behind the norm), "one_part" (one norm over
    everything), "groups" (every head reads group 0)."""
    T = h.shape[0]
    H, VD, N, G, parts = mx["heads"], mx["vdim"], mx["state"], mx["groups"], mx["norm_groups"]
    inner = H * VD
    y = lin(h, W, p + "in")
    z, xbc, dt = y[:, :inner], y[:, inner:2 * inner + 2 * G * N], y[:, 2 * inner + 2 * G * N:]
    if "conv" not in without:
        b = W[p + "conv.b"]
        xbc = silu(causal_conv(xbc, W[p + "conv"], torch.zeros_like(b) if "conv_bias" in without else b))
    x = xbc[:, :inner].reshape(T, H, VD)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    of = torch.zeros(H, dtype=torch.long) if "groups" in without else torch.arange(H) // (H // G)
    B, C = B[:, of], C[:, of]
    dt = softplus(dt + W[p + "dt_bias"].to(F64))
    a = torch.exp(-torch.exp(W[p + "A_log"].to(F64)) * dt)
    if "state" in without:
        a = torch.zeros_like(a)
    o = decay_scan(C, dt[:, :, None] * B, x, a[:, :, None].expand(T, H, N))
    if "skip" not in without:
        o = o + W[p + "D"].to(F64)[None, :, None] * x
    o = o.reshape(T, inner)
    if "z_gate" not in without and "gate_behind" not in without:
        o = o * silu(z)
    n = 1 if "one_part" in without else parts
    o = rms_unit(o.reshape(T, n, inner // n), eps).reshape(T, inner) * W[p + "norm"].to(F64)
    if "gate_behind" in without:
        o = o * silu(z)
    return lin(o, W, p + "o")


# ---------------------------------------------------------------------------------------------- feed-forward and the model
def dense(h, W, p, mlp, without=()):
    """`without`: "limit", "plus_one"."""
    lim = 1e30 if "limit" in without else float(mlp["limit"])
    g, u = torch.clamp(lin(h, W, p + "gate"), max=lim), torch.clamp(lin(h, W, p + "up"), -lim, lim)
    return lin(g * torch.sigmoid(1.702 * g) * (u if "plus_one" in without else u + 1.0), W, p + "down")


def forward(cfg, W, tokens, taps=None, without=()):
    """logits [T, vocab] of one sequence; taps (a list) receives the stream after every layer; `without` bends mechanisms (see the functions above)."""
    eps = float(cfg["norm"]["eps"])
    norm = lambda x, name: layer_norm(x, W[name], W[name + ".b"], eps, without)
    x = W["embed"].to(F64)[torch.as_tensor(list(tokens), dtype=torch.long)] * float(cfg["embedding"]["scale"])
    for il, lc in enumerate(cfg["layers"]):
        p = "l%d." % il
        mix = {"parallel": parallel, "attention": attention, "mamba2": mamba2}[lc["type"]]
        x = x + mix(norm(x, p + "norm1"), W, p + "mix.", lc["mixer"], eps, without)
        if lc.get("mlp"):
            x = x + dense(norm(x, p + "norm2"), W, p + "mlp.", lc["mlp"], without)
        if taps is not None:
            taps.append(x.clone())
    return lin(norm(x, "final.norm"), W, "embed")
