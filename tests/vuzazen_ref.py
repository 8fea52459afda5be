"""Plain, slow restatement of the Vuzazen design in float64 torch, one function per mechanism.

Test infrastructure only: it shares no code with the product path (cortex.llamacpp_amd/), runs on the CPU and
processes whole sequences at once - no cache, no batching, the recurrence token by token.  Weights are a dict
name -> tensor, the configuration is the dict a model's config.json holds.

Notation: x [T, width] the residual stream of one sequence, positions 0 .. T-1; n(y, w) = y / rms(y) * (1 + w), u(y) = y / rms(y).
  embedding:  x_t = scale * E[t] + B[(prev * a + tok * b) mod buckets];  B's last row for the first token
  layer:      x <- x + mixer(n(x, n1));  x <- x + ff(n(x, n2))   (a layer may have no ff)
  mlstm:      q = Wq h / sqrt(dim), k = Wk h, v = Wv h per head;  i = cap tanh((Wi h + bi) / cap),
              f = log sigmoid(cap tanh((Wf h + bf) / cap));  m' = max(f + m, i) from m = 0;
              S' = e^(f+m-m') S + e^(i-m') k v^T,  z' alike with k alone;  o = S'^T q / (max(|z'.q|, e^-m') + 1e-6);
              u(o) per head, times w, times sigmoid(Wg h);  Wo
  latent:     cq = u(Wdq h) wq;  q = Wuq cq per head [dim | rot];  [c | r] = Wdkv h, c <- u(c) wkv;  r and q's rot part turn
              (entry i with entry i + rot/2);  s(i, j) = (q_i.(Wuk c_j) + qr_i.r_j) scale, j <= i;  softmax;  sum of Wuv c_j;
              times sigmoid(Wg h)[head];  Wo
  attention:  q, k, v of H / G / G heads, each channel through a causal convolution of `taps` taps (the last tap at the token itself);
              q <- u(q) wq, k <- u(k) wk over all heads at once;  v <- u(v) per head;  s_h(i, j) = sum_g T[h, g] (q_g,i . k_g,j) scale,
              j <= i;  softmax;  times sigmoid(Wg h)[head];  Wo
  dense ff:   Wdown (silu(Wgate h) * (Wup h))
  experts:    s = sigmoid(Wr h);  the `top` largest s (lower index on a tie);  sum of expert_e(s_e h), each a dense ff
  output:     logits = E n(x, final)
"""
from __future__ import annotations

import torch

F64 = torch.float64


def rms_unit(x, eps):
    """x over its root mean square along the last axis, eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms_unit(x, eps) * (1.0 + w.to(F64))


def lin(x, W, name):
    return x @ W[name].to(F64).T


def silu(z):
    return z * torch.sigmoid(z)


# ---------------------------------------------------------------------------------------------- embedding
def bigram_row(prev, tok, bg):
    """Row of the bigram table for token `tok` behind token `prev` (None: the sequence's first token)."""
    if prev is None:
        return bg["buckets"]
    return (prev * bg["mul_prev"] + tok * bg["mul_cur"]) % bg["buckets"]


def embedding(cfg, W, tokens, without=()):
    """`without`: "bigram"; "first_row" (the first token reads the row of a previous token 0); "previous" (every token reads the first token's row)."""
    em = cfg["embedding"]
    x = W["embed"].to(F64)[torch.as_tensor(tokens, dtype=torch.long)] * float(em["scale"])
    if "bigram" in without:
        return x
    prev = [0 if "first_row" in without else None] + list(tokens[:-1])
    if "previous" in without:
        prev = [None] * len(tokens)
    rows = [bigram_row(p, t, em["bigram"]) for p, t in zip(prev, tokens)]
    return x + W["bigram"].to(F64)[rows]


# ---------------------------------------------------------------------------------------------- mLSTM
def mlstm_gates(zi, zf, cap):
    """Pre-activations (bias included) -> log input gate, log forget gate."""
    f = cap * torch.tanh(zf / cap)
    return cap * torch.tanh(zi / cap), torch.nn.functional.logsigmoid(f)


def mlstm_scan(q, k, v, i, f, floor=True):
    """q, k [T, H, D] (q scaled), v [T, H, VD], i, f [T, H] -> o [T, H, VD].  floor=False leaves e^-m out of the denominator's maximum."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    z = torch.zeros(H, D, dtype=F64)
    m = torch.zeros(H, dtype=F64)
    out = []
    for t in range(T):
        mn = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - mn), torch.exp(i[t] - mn)
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + take[:, None] * k[t]
        m = mn
        zq = (z * q[t]).sum(-1).abs()
        den = (torch.maximum(zq, torch.exp(-m)) if floor else zq) + 1e-6
        out.append((S * q[t][:, :, None]).sum(1) / den[:, None])
    return torch.stack(out)


def mlstm(h, W, p, mx, eps, without=()):
    """`without`: "state" (every token sees only itself), "cap" (the gates' pre-activations uncapped), "floor", "gate"."""
    T = h.shape[0]
    H, D, VD = mx["heads"], mx["dim"], mx["vdim"]
    q = lin(h, W, p + "q").reshape(T, H, D) * D ** -0.5
    k = lin(h, W, p + "k").reshape(T, H, D)
    v = lin(h, W, p + "v").reshape(T, H, VD)
    cap = 1e6 if "cap" in without else float(mx["gate_cap"])
    i, f = mlstm_gates(lin(h, W, p + "i") + W[p + "i.b"].to(F64), lin(h, W, p + "f") + W[p + "f.b"].to(F64), cap)
    if "state" in without:
        o = torch.cat([mlstm_scan(q[t:t + 1], k[t:t + 1], v[t:t + 1], i[t:t + 1], f[t:t + 1]) for t in range(T)])
    else:
        o = mlstm_scan(q, k, v, i, f, "floor" not in without)
    o = rms_unit(o, eps).reshape(T, H * VD) * W[p + "norm"].to(F64)
    if "gate" not in without:
        o = o * torch.sigmoid(lin(h, W, p + "g"))
    return lin(o, W, p + "o")


# ---------------------------------------------------------------------------------------------- latent attention
def turn_halves(x, base):
    """x [T, ..., D] of positions 0 .. T-1: entry i < D/2 pairs with entry i + D/2 and turns by p * base^(-2i/D)."""
    T, D = x.shape[0], x.shape[-1]
    half = D // 2
    freq = float(base) ** (-2.0 * torch.arange(half, dtype=F64) / D)
    ang = (torch.arange(T, dtype=F64)[:, None] * freq[None, :]).reshape((T,) + (1,) * (x.dim() - 2) + (half,))
    c, s = torch.cos(ang), torch.sin(ang)
    a, b = x[..., :half], x[..., half:]
    return torch.cat([a * c - b * s, b * c + a * s], dim=-1)


def causal_softmax(s):
    T = s.shape[0]
    seen = torch.ones(T, T, dtype=torch.bool).tril()
    return torch.softmax(s.masked_fill(~seen, float("-inf")), -1)


def latent_attention(h, W, p, mx, eps, without=()):
    """`without`: "rotation", "latent_norm", "gate"."""
    T = h.shape[0]
    H, D, R, VD, KR = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    cq = rms_unit(lin(h, W, p + "dq"), eps) * W[p + "dq.norm"].to(F64)
    q = lin(cq, W, p + "uq").reshape(T, H, D + R)
    down = lin(h, W, p + "dkv")
    c = (down[:, :KR] if "latent_norm" in without else rms_unit(down[:, :KR], eps)) * W[p + "dkv.norm"].to(F64)
    qr, r = q[..., D:], down[:, KR:]
    if R and "rotation" not in without:
        qr, r = turn_halves(qr, mx["rot"]["base"]), turn_halves(r, mx["rot"]["base"])
    k = lin(c, W, p + "uk").reshape(T, H, D)
    v = lin(c, W, p + "uv").reshape(T, H, VD)
    g = torch.sigmoid(lin(h, W, p + "g"))
    heads = []
    for a in range(H):
        w = causal_softmax((q[:, a, :D] @ k[:, a].T + qr[:, a] @ r.T) * float(mx["scale"]))
        o = w @ v[:, a]
        heads.append(o if "gate" in without else o * g[:, a:a + 1])
    return lin(torch.cat(heads, -1), W, p + "o")


# ---------------------------------------------------------------------------------------------- attention with mixed scores
def causal_conv(u, w):
    """u [T, C], w [C, taps]: the last tap meets the token itself, the ones before it the tokens before; zeros in front of the sequence."""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    return sum(pad[j:j + T] * w[:, j].to(F64) for j in range(taps))


def attention(h, W, p, mx, eps, without=()):
    """`without`: "conv", "talk" (heads' scores unmixed), "talk_turned" (mixed with the transpose), "qk_norm", "v_norm", "gate"."""
    T = h.shape[0]
    H, G, D, VD = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (lin(h, W, p + n) if "conv" in without else causal_conv(lin(h, W, p + n), W[p + n + ".conv"]) for n in "qkv")
    if "qk_norm" not in without:
        q = rms_unit(q, eps) * W[p + "q.norm"].to(F64)
        k = rms_unit(k, eps) * W[p + "k.norm"].to(F64)
    q, k, v = q.reshape(T, H, D), k.reshape(T, G, D), v.reshape(T, G, VD)
    if "v_norm" not in without:
        v = rms_unit(v, eps)
    raw = torch.stack([(q[:, a] @ k[:, a // (H // G)].T) * float(mx["scale"]) for a in range(H)])
    talk = W[p + "talk"].to(F64)
    talk = torch.eye(H, dtype=F64) if "talk" in without else talk.T if "talk_turned" in without else talk
    mixed = (talk @ raw.reshape(H, T * T)).reshape(H, T, T)
    g = torch.sigmoid(lin(h, W, p + "g"))
    heads = []
    for a in range(H):
        o = causal_softmax(mixed[a]) @ v[:, a // (H // G)]
        heads.append(o if "gate" in without else o * g[:, a:a + 1])
    return lin(torch.cat(heads, -1), W, p + "o")


# ---------------------------------------------------------------------------------------------- feed-forwards
def dense(h, W, p):
    return lin(silu(lin(h, W, p + "gate")) * lin(h, W, p + "up"), W, p + "down")


def route(z, top):
    """z [T, E] router logits -> (ids [T, top], weights [T, top]); ties go to the lower index."""
    s = torch.sigmoid(z)
    ids = torch.stack([torch.tensor(sorted(range(s.shape[1]), key=lambda e: (-float(s[t, e]), e))[:top]) for t in range(s.shape[0])])
    return ids, s.gather(1, ids)


def experts(h, W, p, mlp, without=()):
    """`without`: "weight" (the experts read h itself), "weight_in" (the weight multiplies the expert's output)."""
    ids, w = route(lin(h, W, p + "router"), mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(ids.shape[1]):
            pe, x, wt = p + "e%d." % int(ids[t, j]), h[t:t + 1], w[t, j]
            if "weight" in without:
                out[t] += dense(x, W, pe)[0]
            elif "weight_in" in without:
                out[t] += wt * dense(x, W, pe)[0]
            else:
                out[t] += dense(wt * x, W, pe)[0]
    return out


# ---------------------------------------------------------------------------------------------- the model
def forward(cfg, W, tokens, taps=None, without=()):
    """logits [T, vocab] of one sequence; taps (a list) receives the stream after every layer; `without` bends mechanisms (see the functions above)."""
    eps = float(cfg["norm"]["eps"])
    x = embedding(cfg, W, list(tokens), without)
    for il, lc in enumerate(cfg["layers"]):
        p = "l%d." % il
        h = norm(x, W[p + "norm1"], eps)
        mix = {"mlstm": mlstm, "latent_attention": latent_attention, "attention": attention}[lc["type"]]
        x = x + mix(h, W, p + "mix.", lc["mixer"], eps, without)
        if lc.get("mlp"):
            h = norm(x, W[p + "norm2"], eps)
            x = x + (dense(h, W, p + "mlp.") if lc["mlp"]["kind"] == "dense" else experts(h, W, p + "mlp.", lc["mlp"], without))
        if taps is not None:
            taps.append(x.clone())
    return lin(norm(x, W["final.norm"], eps), W, "embed")
