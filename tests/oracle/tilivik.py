"""Plain, slow restatement of the Tilivik design, one function per
mechanism, used as ground truth by the tests.

Everything is computed token by token with explicit loops over heads and
experts, in whatever float type the weights are given in (the tests use
float64).  Nothing here is shared with scaffold/.

A sequence of hidden vectors is a (T, width) tensor; weights are a dict
of tensors keyed by their checkpoint names.
"""

import math

import torch


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms(x, eps):
    """x over its root mean square along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


# ------------------------------------------------------------- embedding
def bigram_row(prev, tok, spec):
    """Row of the pair table; prev None: the sequence's first token."""
    if prev is None:
        return spec["buckets"]
    return (prev * spec["mul_prev"] + tok * spec["mul_cur"]) % spec["buckets"]


def sinusoid(p, width):
    """Position p's vector: sine and cosine of slower and slower turns."""
    out = []
    for c in range(width):
        angle = p * 10000.0 ** (-2 * (c // 2) / width)
        out.append(math.cos(angle) if c % 2 else math.sin(angle))
    return torch.tensor(out, dtype=torch.float64)


def embedding(cfg, w, tokens):
    spec, rows = cfg["embedding"]["bigram"], []
    for p, tok in enumerate(tokens):
        prev = tokens[p - 1] if p else None
        pair = w["bigram"][bigram_row(prev, tok, spec)]
        rows.append(w["embed"][tok] + pair
                    + sinusoid(p, cfg["width"]).to(pair.dtype))
    return torch.stack(rows)


def token_shift(h, mix):
    """Blend every vector with the one before it (zeros before the first)."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mix


# -------------------------------------------------------------- recurrences
def lightning_mixer(h, w, p, mx, eps):
    T, H, d, e = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = silu(h @ w[p + "q"].T).view(T, H, d)
    k = silu(h @ w[p + "k"].T).view(T, H, d)
    v = silu(h @ w[p + "v"].T).view(T, H, e)
    o = torch.zeros(T, H, e, dtype=h.dtype)
    for a in range(H):
        S = torch.zeros(d, e, dtype=h.dtype)
        for t in range(T):
            S = mx["decay"][a] * S + torch.outer(k[t, a], v[t, a])
            o[t, a] = S.T @ q[t, a]
    y = rms(o.reshape(T, H * e), eps) * w[p + "norm"]
    return (y * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def channel_decay(z, tau):
    return sigmoid(z) ** (1 / tau)


def gla_mixer(h, w, p, mx, eps):
    """Linear attention whose state rows decay each by their own factor."""
    T, H, d, e = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[p + "q"].T * d ** -0.5).view(T, H, d)
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, e)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = channel_decay(z, mx["tau"]).view(T, H, d)
    o = torch.zeros(T, H, e, dtype=h.dtype)
    for a in range(H):
        S = torch.zeros(d, e, dtype=h.dtype)
        for t in range(T):
            S = alpha[t, a].unsqueeze(1) * S + torch.outer(k[t, a], v[t, a])
            o[t, a] = S.T @ q[t, a]
    y = (rms(o, eps) * w[p + "norm"]).reshape(T, H * e)
    return (y * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---------------------------------------------------------------- attention
def bucket(n, rows, far):
    """Row of the bias table for distance n: exact at first, then by its
    logarithm, the last row from `far` on."""
    half = rows // 2
    if n < half:
        return n
    steps = math.log(n / half) / math.log(far / half) * (rows - half)
    return min(rows - 1, half + math.floor(steps))


def visible(i, j, mask):
    return j <= i and (not mask.get("size") or i - j < mask["size"]
                       or j < mask.get("keep_first", 0))


def window_attention(q, k, v, rel, mx, pos0=0):
    """q (n,H,d) at positions pos0.., k (T,G,d), v (T,G,e) from position 0
    -> (n,H,e)."""
    n, H, _ = q.shape
    rep = H // k.shape[1]
    mask, cap = mx.get("mask") or {}, mx["softcap"]
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for r in range(n):
        i = pos0 + r
        seen = [j for j in range(i + 1) if visible(i, j, mask)]
        rows = [bucket(i - j, rel.shape[0], mx["bias_max"]) for j in seen]
        for h in range(H):
            s = k[seen, h // rep] @ q[r, h] * mx["scale"]
            s = cap * torch.tanh(s / cap) + rel[rows, h]
            out[r, h] = torch.softmax(s, 0) @ v[seen, h // rep]
    return out


def attention_mixer(h, w, p, mx, eps):
    T, H, G = h.shape[0], mx["heads"], mx["kv_heads"]
    q = (h @ w[p + "q"].T).view(T, H, mx["dim"])
    k = (h @ w[p + "k"].T).view(T, G, mx["dim"])
    v = rms((h @ w[p + "v"].T).view(T, G, mx["vdim"]), eps)
    o = window_attention(q, k, v, w[p + "rel"], mx).reshape(T, -1)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, w, p, mx, eps):
    return (mx["left_scale"] * attention_mixer(h, w, p + "left.", mx["left"], eps)
            + mx["right_scale"] * gla_mixer(h, w, p + "right.", mx["right"], eps))


# ------------------------------------------------------------- feed-forward
def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def table_moe(h, w, p, tokens):
    """Experts by token id, equal weights."""
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        chosen = w[p + "table"][tok].long().tolist()
        for e in chosen:
            out[t] += expert(h[t], w, f"{p}e{e}.") / len(chosen)
    return out


# -------------------------------------------------------------------- model
def layer_order(cfg):
    """(layer, number of the pass it begins or None) in running order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    lo, hi = loop["start"], loop["stop"]
    span = [(i, t if i == lo else None) for t in range(loop["times"])
            for i in range(lo, hi)]
    return ([(i, None) for i in range(lo)] + span
            + [(i, None) for i in range(hi, n)])


MIXERS = {"lightning": lightning_mixer, "parallel": parallel_mixer}


def forward(cfg, w, tokens, collect=None):
    """Logits (T, vocab) of one sequence; `collect` gets the residual
    stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x = first = embedding(cfg, w, tokens)
    for i, begins in layer_order(cfg):
        if begins is not None:
            if begins > 0:
                x = x + first
            x = x + w["loop.step"][begins]
        L, p = cfg["layers"][i], f"l{i}."
        h = token_shift(rms(x, eps) * w[p + "norm1"], w[p + "shift"])
        x = x + MIXERS[L["type"]](h, w, p + "mix.", L["mixer"], eps)
        if L["mlp"] is not None:
            x = x + table_moe(rms(x, eps) * w[p + "norm2"], w, p + "mlp.",
                              tokens)
        if collect is not None:
            collect.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
