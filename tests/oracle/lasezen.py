"""Plain, slow restatement of the Lasezen design, one function per
mechanism, used as ground truth by the tests.

Everything is computed token by token with explicit loops over heads
and keys, in whatever float type the weights are given in (the tests
use float64).  Nothing here is shared with scaffold/.

A sequence of hidden vectors is a (T, width) tensor; weights are a dict
of tensors keyed by their checkpoint names.
"""

import math

import torch


def rms(x, eps, weight=None):
    """x over its root mean square along the last dimension."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def layer_norm(x, weight, bias, eps):
    mu = x.mean(-1, keepdim=True)
    var = ((x - mu) ** 2).mean(-1, keepdim=True)
    return (x - mu) / torch.sqrt(var + eps) * weight + bias


def gelu(z):
    return z * 0.5 * (1 + torch.erf(z / math.sqrt(2.0)))


def dense_ff(h, w_up, w_down):
    return gelu(h @ w_up.T) @ w_down.T


def rotate_half(x, pos, base, dims):
    """x (d,) at position pos: coordinate i and i + dims/2 turn together
    by pos * base^(-2i/dims); coordinates from dims on stay."""
    y = x.clone()
    half = dims // 2
    for i in range(half):
        a = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = x[i], x[i + half]
        y[i] = u * c - v * s
        y[i + half] = v * c + u * s
    return y


def visible(i, j, size):
    """Key j for query i under chunks of `size` (0: every earlier key)."""
    return j <= i and (not size or i // size == j // size)


def sink_attention(q, k, v, scale, size, sink):
    """q (T,H,d), k (T,G,d), v (T,G,e), sink (H,) or None -> (T,H,e)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        js = [j for j in range(i + 1) if visible(i, j, size)]
        for h in range(H):
            g = h // (H // G)
            s = torch.stack([(q[i, h] * k[j, g]).sum() * scale for j in js])
            top = s.max()
            if sink is not None:
                top = torch.maximum(top, sink[h])
            e = torch.exp(s - top)
            den = e.sum()
            if sink is not None:
                den = den + torch.exp(sink[h] - top)
            for w, j in zip(e, js):
                out[i, h] += w / den * v[j, g]
    return out


def attention_mixer(h, w, p, mx, eps):
    T, H, G = h.shape[0], mx["heads"], mx["kv_heads"]
    q = (h @ w[p + "q"].T).view(T, H, mx["dim"])
    k = (h @ w[p + "k"].T).view(T, G, mx["dim"])
    v = (h @ w[p + "v"].T).view(T, G, mx["vdim"])
    q = rms(q, eps, w[p + "q.norm"])
    k = rms(k, eps, w[p + "k.norm"])
    o = sink_attention(q, k, v, mx["scale"], mx["mask"]["size"], w[p + "sink"])
    return o.reshape(T, -1) @ w[p + "o"].T


def retention_core(q, k, v, decay, state=None):
    """q, k (T,H,d), v (T,H,e), decay list of H floats; the recurrence
    S <- decay * S + k v^T, o = S^T q.  Returns (o (T,H,e), S (H,d,e))."""
    T, H, d = q.shape
    e = v.shape[2]
    S = torch.zeros(H, d, e, dtype=q.dtype) if state is None else state.clone()
    o = torch.zeros(T, H, e, dtype=q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + torch.outer(k[t, h], v[t, h])
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def retention_mixer(h, w, p, mx, eps):
    T, H = h.shape[0], mx["heads"]
    q = (h @ w[p + "q"].T).view(T, H, mx["dim"])
    k = (h @ w[p + "k"].T).view(T, H, mx["dim"])
    v = (h @ w[p + "v"].T).view(T, H, mx["vdim"])
    rot = mx["rot"]
    for t in range(T):
        for a in range(H):
            q[t, a] = rotate_half(q[t, a], t, rot["base"], rot["dims"])
            k[t, a] = rotate_half(k[t, a], t, rot["base"], rot["dims"])
    k = k * mx["dim"] ** -0.5
    o, _ = retention_core(q, k, v, mx["decay"])
    o = rms(o, eps).reshape(T, -1)
    z = h @ w[p + "g"].T
    return (o * (z / (1 + torch.exp(-z)))) @ w[p + "o"].T


def layer_order(cfg):
    """Indices of the layers in the order they run."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return list(range(n))
    body = list(range(lp["start"], lp["stop"]))
    return (list(range(lp["start"])) + body * lp["times"]
            + list(range(lp["stop"], n)))


def forward(cfg, w, tokens, collect=None):
    """Logits (T, vocab) of one sequence; `collect` gets the residual
    stream after every layer run."""
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.tensor(tokens)].clone()

    def norm(name, y):
        return layer_norm(y, w[name], w[name + ".b"], eps)

    for i in layer_order(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        mixer = {"attention": attention_mixer,
                 "retention": retention_mixer}[L["type"]]
        y = mixer(norm(p + "norm1", x), w, p + "mix.", L["mixer"], eps)
        x = x + m * norm(p + "norm1b", y)
        if L["mlp"] is not None:
            y = dense_ff(norm(p + "norm2", x), w[p + "mlp.up"],
                         w[p + "mlp.down"])
            x = x + m * norm(p + "norm2b", y)
        if collect is not None:
            collect.append(x.clone())
    return norm("final.norm", x) @ w["head"].T
