"""Ops of the mixer-stack models (paged, tied, window and latent attention,
retention, gated linear attention, state-space and matrix-memory
recurrences, routed experts, embeddings, residual norms).  GPU tensors run
the HIP kernels of csrc/lm, required; CPU tensors run the plain float32
forms below, which the CPU tests use.
"""

from __future__ import annotations

import math
from typing import NamedTuple, Optional, Tuple

import torch
import torch.nn.functional as F

from .backend import require_lm_ext


def rope_tables_exact(seq_len: int, dims: int, base: float, device,
                      scaling: Optional[dict] = None
                      ) -> Tuple[torch.Tensor, torch.Tensor]:
    """cos/sin (seq_len, dims/2) in float32, angles in float64: the table
    entries carry no error of the angle, however long the sequence.

    scaling: YaRN (Peng et al., "YaRN: Efficient Context Window Extension
    of Large Language Models"): pairs that turn fewer than `slow` times
    over `original` positions are slowed by `factor`, those that turn more
    than `fast` times keep their speed, the ones between are blended; cos
    and sin grow by 0.1 ln(factor) + 1."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    freq = float(base) ** (-2.0 * i / dims)
    mult = 1.0
    if scaling:
        def pair_turning(n):         # (real) index of the pair with n turns
            return (dims * math.log(scaling["original"] / (2 * math.pi * n))
                    / (2 * math.log(base)))

        lo = max(math.floor(pair_turning(scaling["fast"])), 0)
        hi = min(math.ceil(pair_turning(scaling["slow"])), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
        freq = freq / scaling["factor"] * ramp + freq * (1 - ramp)
        mult = 0.1 * math.log(scaling["factor"]) + 1.0
    ang = torch.outer(torch.arange(seq_len, dtype=torch.float64), freq)
    return ((mult * ang.cos()).float().to(device).contiguous(),
            (mult * ang.sin()).float().to(device).contiguous())


def decay_tables(decay, tile: int, device) -> Tuple[torch.Tensor, torch.Tensor]:
    """(powers (H, tile+1) = decay^n, decays (H, 2) as float + remainder)."""
    d = torch.tensor(decay, dtype=torch.float64)
    n = torch.arange(tile + 1, dtype=torch.float64)
    pows = d.unsqueeze(1) ** n
    hi = d.float()
    lo = (d - hi.double()).float()
    return (pows.float().to(device).contiguous(),
            torch.stack([hi, lo], 1).to(device).contiguous())


class Parts(NamedTuple):
    """A sublayer's output as a weighted sum that is still to be taken:
    y (T, n, W), weights (T, n) float32."""
    y: torch.Tensor
    weights: torch.Tensor

    def total(self) -> torch.Tensor:
        return (self.y.float() * self.weights.unsqueeze(2)).sum(1)


# A norm is given as its parameters: (weight,) is an RMS norm (its weight may
# be a single number), (weight, bias or None) a layer norm, (weight, bias, alpha) a dynamic tanh, None
# leaves its input as it is.
def _norm(x, p, eps):
    if p is None:
        return x.float()
    if len(p) == 1:
        return _rms(x, eps, p[0])
    if len(p) == 3:
        w, b, alpha = (t.float() for t in p)
        return torch.tanh(alpha * x.float()) * w + b
    w, b = p
    return F.layer_norm(x.float(), (x.shape[-1],), w.float(),
                        None if b is None else b.float(), eps)


def _wba(p):
    """weight, bias, alpha, whether it is an RMS norm."""
    p = p or ()
    return (*(*p, None, None, None)[:3], len(p) == 1)


def _yw(y):
    return (y.y, y.weights) if isinstance(y, Parts) else (y, None)


def _advance(x, y, post, mult, eps):
    if y is None:
        return x
    if isinstance(y, Parts):
        y = y.total()
    return x + mult * _norm(y, post, eps)


def embed_norm(tokens, embed, norm, eps, pos=None, positions=None):
    """Residual stream x (float32) of the tokens and its first norm.
    positions: a table of vectors to add, row pos[t] for token t."""
    if embed.is_cuda:
        return require_lm_ext().embed_norm(tokens, embed, pos, positions,
                                           *_wba(norm), eps)
    x = embed[tokens].float()
    if positions is not None:
        x = x + positions[pos.long()].float()
    return x, _norm(x, norm, eps).to(embed.dtype)


def turn_rates(width: int, base: float, device) -> torch.Tensor:
    """(width/2, rounded up) float64: what entries 2i and 2i+1 of a
    sinusoidal position vector turn by per position, base^(-2i/width), in
    whole turns."""
    i = torch.arange(-(-width // 2), dtype=torch.float64)
    return (float(base) ** (-2.0 * i / width) / (2 * math.pi)).to(device)


def _before(t, plan, state):
    """Rows t (T, ...) of a ragged batch moved down by one token: each gets
    its predecessor's, a sequence's first one zeros, a portion's first one
    what `state` kept; then state keeps the portions' last rows."""
    out = torch.zeros_like(t)
    for r0, n, p0, s in _portions(plan):
        out[r0 + 1:r0 + n] = t[r0:r0 + n - 1]
        if p0:
            out[r0] = state[s]
        state[s] = t[r0 + n - 1]
    return out


def stream_embed(plan, embed, *, rates=None, pairs=None, mul=(0, 0),
                 last=None):
    """Residual stream x (float32) of a ragged batch's tokens: their
    embeddings, plus (rates: turn_rates) sinusoidal position vectors, plus
    (pairs: a table) row (previous * mul[0] + token * mul[1]) mod (rows - 1),
    for a sequence's first token the last row.  last (slots,) int64: the
    token before, kept per slot."""
    if embed.is_cuda:
        return require_lm_ext().stream_embed(
            plan.tokens, embed, plan.pos, plan.slot, plan.tiles, plan.seqs,
            plan.n_dec, rates, pairs, *mul, last)
    x = embed[plan.tokens].float()
    if pairs is not None:
        n = pairs.shape[0] - 1
        row = (_before(plan.tokens, plan, last) * mul[0]
               + plan.tokens * mul[1]) % n
        x = x + pairs[row.masked_fill(plan.pos == 0, n)].float()
    if rates is not None:
        turns = plan.pos.double().unsqueeze(1) * rates
        ang = 2 * math.pi * (turns - turns.floor())
        x = x + torch.stack([ang.sin(), ang.cos()], 2).flatten(1)[
            :, :x.shape[1]].float()
    return x


def shift_norm(x, y, mult, nxt, eps, plan, *, shift=None, state=None, add=None,
               step=None):
    """A new stream x + mult * y + add + step (y: (T, W), Parts or None; add:
    a float32 stream or None; step: a vector or None) and its norm, which
    (shift: a vector) is blended with the previous token's, h + (h' - h) *
    shift.  state (slots, W) keeps a sequence's last h, unblended; None:
    nobody looks back at these."""
    if x.is_cuda:
        return require_lm_ext().shift_norm(
            x, *_yw(y), mult, *_wba(nxt), eps, plan.pos, plan.slot, plan.tiles,
            plan.seqs, plan.n_dec, shift, state, add, step)
    z = x.clone() if y is None else _advance(x, y, None, mult, eps)
    if add is not None:
        z = z + add
    if step is not None:
        z = z + step.float()
    h = _norm(z, nxt, eps)
    if shift is not None:
        h = h + (_before(h, plan, state) - h) * shift.float()
    return z, h.to(nxt[0].dtype)


def residual_norm(x, y, post, mult, nxt, eps, rows=None, store_x=True):
    """x += mult * norm(y; post), then norm(x; nxt) of `rows` (None: all).
    y: (T, W), Parts of one, or None."""
    if x.is_cuda:
        return require_lm_ext().residual_norm(
            x, *_yw(y), *_wba(post), mult, *_wba(nxt), rows, eps, store_x)
    z = _advance(x, y, post, mult, eps)
    if store_x and y is not None:
        x.copy_(z)
    if rows is not None:
        z = z[rows.long()]
    return _norm(z, nxt, eps).to((_yw(y)[0] if nxt is None else nxt[0]).dtype)


def residual_concat(x, y, post, mult, eps, tokens, embed):
    """x += mult * norm(y; post) as in residual_norm, then (T, 2W): the
    stream beside the tokens' embeddings, both in the embeddings' type."""
    if x.is_cuda:
        return require_lm_ext().residual_concat(
            x, *_yw(y), *_wba(post), mult, tokens, embed, eps)
    x.copy_(_advance(x, y, post, mult, eps))
    return torch.cat([x.to(embed.dtype), embed[tokens]], 1)


def replace_norm(x, y, step, nxt, eps):
    """x <- y + step (a vector), then norm(x; nxt)."""
    if x.is_cuda:
        return require_lm_ext().replace_norm(x, y, step, *_wba(nxt), eps)
    x.copy_(y.float() + step.float())
    return _norm(x, nxt, eps).to(step.dtype)


def softcap(x, cap):
    """cap * tanh(x / cap), in float32."""
    if x.is_cuda:
        return require_lm_ext().softcap(x, cap)
    return cap * torch.tanh(x.float() / cap)


def geglu_tanh(gu):
    """gelu(g) * u of rows [g | u], the tanh form of GELU."""
    if gu.is_cuda:
        return require_lm_ext().geglu_tanh(gu)
    g, u = gu.float().chunk(2, -1)
    return (F.gelu(g, approximate="tanh") * u).to(gu.dtype)


def clamped_glu(gu, limit, alpha, shift):
    """g sigmoid(alpha g) (u + shift) of rows [g | u], g cut off above
    `limit`, u on both sides."""
    if gu.is_cuda:
        return require_lm_ext().clamped_glu(gu, limit, alpha, shift)
    g, u = gu.float().chunk(2, -1)
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(alpha * g) * (u + shift)).to(gu.dtype)


def gelu_erf(x):
    if x.is_cuda:
        return require_lm_ext().gelu_erf(x)
    return F.gelu(x.float()).to(x.dtype)


def linear(x, w, b=None):
    from . import linear as f      # the framework's matrix product

    return f(x, w, b)


def linear_f32(x, w):
    """linear() with a float32 result, not rounded to the inputs' type."""
    if x.is_cuda and x.dtype == torch.bfloat16:
        return torch.mm(x, w.t(), out_dtype=torch.float32)
    return linear(x, w).float()


def _portions(plan):
    """(first row, rows, first position, slot) of every sequence's part."""
    pos, slot = plan.pos.tolist(), plan.slot.tolist()
    out = [(r, 1, pos[r], slot[r]) for r in range(plan.n_dec) if slot[r] >= 0]
    tiles = plan.tiles.tolist()
    for t0, n, p0, s in plan.seqs.tolist():
        rows = sum(tiles[t][1] for t in range(t0, t0 + n))
        out.append((tiles[t0][0], rows, p0, s))
    return out


def _rms(x, eps, w=None):
    x = x.float()
    y = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w.float()


def _attend(q, k, v, pos, j, *, size, scale, sink=None, slopes=None,
            keep=None, softcap=0.0, bias=None):
    """q (n, H, d) at positions pos over keys k, values v (m, G, .) at
    positions j -> (n, H, e), float32.  sink: (H,) scores without a value,
    or None; slopes: (H,) off the scores per step of distance, or None; size:
    chunk length or (keep is a number) window length beside which the first
    `keep` tokens stay visible; bias: (H, n) added per distance, the last
    column from there on."""
    n, H, _ = q.shape
    rep = H // k.shape[1]
    kk = k.float().repeat_interleave(rep, 1)
    vv = v.float().repeat_interleave(rep, 1)
    sc = torch.einsum("ihd,jhd->hij", q.float(), kk) * scale
    if slopes is not None:
        dist = (pos[:, None] - j[None]).float()
        sc = sc - slopes.float().view(-1, 1, 1) * dist
    if softcap:
        sc = softcap * torch.tanh(sc / softcap)
    if bias is not None:
        dist = (pos[:, None] - j[None]).clamp(0, bias.shape[1] - 1)
        sc = sc + bias[:, dist]
    see = j[None] <= pos[:, None]
    if size and keep is not None:
        see &= (pos[:, None] - j[None] < size) | (j[None] < keep)
    elif size:
        see &= j[None] // size == pos[:, None] // size
    sc = sc.masked_fill(~see, float("-inf"))
    if sink is not None:
        sc = torch.cat([sc, sink.float().view(-1, 1, 1).expand(-1, n, 1)], 2)
    p = torch.softmax(sc, dim=2)[:, :, :j.numel()]
    return torch.einsum("hij,jhe->ihe", p, vv)


def paged_attention(qkv, cache, run, plan, *, heads, q_norm, k_norm, sink,
                    size, scale, eps, slopes=None):
    """Attention of a ragged batch; appends its keys and values to run
    `run` of the cache.  qkv rows are [heads*dim | kv*dim | kv*vdim];
    q_norm, k_norm: per-head RMS weights or None; sink: (heads,) added to
    the softmax denominator, or None; size: chunk length, 0 for plain
    causal; slopes: (heads,) float32 taken off a score per step of distance,
    or None.  Returns (rows, heads * vdim)."""
    kc, vc = cache.k[run], cache.v[run]
    if qkv.is_cuda:
        return require_lm_ext().paged_attention(
            qkv, kc, vc, cache.table, plan.pos, plan.slot, plan.tiles,
            plan.n_dec, q_norm, k_norm, sink, slopes, heads, size, scale, eps,
            cache.max_len)
    G, page, dim, vdim = kc.shape[1], kc.shape[2], kc.shape[3], vc.shape[3]
    q, k, v = torch.split(qkv, [heads * dim, G * dim, G * vdim], dim=1)
    q, k, v = (q.reshape(-1, heads, dim), k.reshape(-1, G, dim),
               v.reshape(-1, G, vdim))
    if q_norm is not None:
        q = _rms(q, eps, q_norm).to(qkv.dtype)
    if k_norm is not None:
        k = _rms(k, eps, k_norm).to(qkv.dtype)
    out = torch.zeros(qkv.shape[0], heads, vdim, dtype=qkv.dtype)
    for r0, n, p0, s in _portions(plan):
        i = torch.arange(p0, p0 + n)
        cell = cache.table[s].long()[i // page]
        kc[cell, :, i % page] = k[r0:r0 + n]
        vc[cell, :, i % page] = v[r0:r0 + n]
        j = torch.arange(p0 - p0 % size if size else 0, p0 + n)
        cell = cache.table[s].long()[j // page]
        out[r0:r0 + n] = _attend(
            q[r0:r0 + n], kc[cell, :, j % page], vc[cell, :, j % page], i, j,
            size=size, scale=scale, sink=sink, slopes=slopes).to(qkv.dtype)
    return out.reshape(qkv.shape[0], heads * vdim)


def distance_bias(rel: torch.Tensor, far: int) -> torch.Tensor:
    """(heads, far + 1) float32: a learned table rel (rows, heads) laid out
    by distance.  The first half of the rows belongs to the distances below
    rows/2 one by one, the others share what follows up to `far` by its
    logarithm (Raffel et al., "Exploring the Limits of Transfer Learning with
    a Unified Text-to-Text Transformer"); the last one also has all beyond."""
    rows = rel.shape[0]
    half = rows // 2

    def row(n):
        if n < half:
            return n
        t = math.log(n / half) / math.log(far / half)
        return min(rows - 1, half + math.floor(t * (rows - half)))

    pick = torch.tensor([row(n) for n in range(far + 1)], device=rel.device)
    return rel.detach()[pick].float().t().contiguous()


def window_attention(x, col, out, out_col, cache, run, plan, *, heads, bias,
                     softcap, size, keep, scale, out_scale, eps):
    """Attention of a ragged batch over the last `size` tokens (0: all) and
    the first `keep`; appends its keys and values to run `run` of the cache.
    x's columns from `col` on are [q | k | v | gate]; each head's value is
    divided by its root mean square.  Scores are capped (softcap, 0: not),
    then take bias (heads, n) by distance.  The result, times the gate's
    sigmoid and out_scale, goes to out's columns from out_col on."""
    kc, vc = cache.k[run], cache.v[run]
    if x.is_cuda:
        return require_lm_ext().window_attention(
            x, col, out, out_col, kc, vc, cache.table, plan.pos, plan.slot,
            plan.tiles, plan.n_dec, bias, softcap, heads, size, keep, scale,
            out_scale, eps, cache.max_len)
    G, page, dim, vdim = kc.shape[1], kc.shape[2], kc.shape[3], vc.shape[3]
    q, k, v, g = torch.split(
        x[:, col:col + heads * (dim + vdim) + G * (dim + vdim)],
        [heads * dim, G * dim, G * vdim, heads * vdim], dim=1)
    q, k = q.reshape(-1, heads, dim), k.reshape(-1, G, dim)
    v = _rms(v.reshape(-1, G, vdim), eps).to(x.dtype)
    for r0, n, p0, s in _portions(plan):
        i = torch.arange(p0, p0 + n)
        cell = cache.table[s].long()[i // page]
        kc[cell, :, i % page] = k[r0:r0 + n]
        vc[cell, :, i % page] = v[r0:r0 + n]
        j = torch.arange(p0 + n)
        if size:
            j = j[(j < keep) | (j > p0 - size)]
        cell = cache.table[s].long()[j // page]
        o = _attend(q[r0:r0 + n], kc[cell, :, j % page], vc[cell, :, j % page],
                    i, j, size=size, keep=keep, scale=scale, softcap=softcap,
                    bias=bias).reshape(n, heads * vdim)
        o = o * torch.sigmoid(g[r0:r0 + n].float()) * out_scale
        out[r0:r0 + n, out_col:out_col + heads * vdim] = o.to(x.dtype)


def tied_attention(x, cache, run, plan, *, heads, q_norm, k_norm, temp, slopes,
                   sink, gated, size, scale, eps):
    """Attention of a ragged batch whose values are its keys, as they are
    before their norm; appends them to run `run` of the cache, each token's
    beside the factor that norms them.  Rows of x are [q | k | gate];
    q_norm, k_norm: weights of RMS norms over all heads of a row; temp:
    (coef, every), q takes 1 + coef ln(floor((p + 1) / every) + 1) at
    position p, or None; slopes as in paged_attention; sink: the score, of
    every head, of a sink without a value, or None; gated: the sigmoid of
    the last heads*dim columns multiplies the result.

    The cache is half of what keys and values would take: a score is the
    query, times the key weights, with the cached row, times its factor."""
    kc, kf = cache.k[run], cache.v[run]
    coef, every = temp or (0.0, 0)
    if x.is_cuda:
        return require_lm_ext().tied_attention(
            x, kc, kf, cache.table, plan.pos, plan.slot, plan.tiles,
            plan.n_dec, q_norm, k_norm, slopes, sink, coef, every, gated,
            heads, size, scale, eps, cache.max_len)
    G, page, dim = kc.shape[1:]
    rows = x.shape[0]
    q, k, g = torch.split(x, [heads * dim, G * dim,
                              x.shape[1] - (heads + G) * dim], dim=1)
    qn = _rms(q, eps, q_norm)
    if every:
        t = torch.div(plan.pos + 1, every, rounding_mode="floor") + 1
        qn = qn * (1 + coef * torch.log(t.float())).unsqueeze(1)
    kw = k_norm.float().view(G, 1, dim).expand(G, heads // G, dim)
    q = (qn.view(rows, G, heads // G, dim) * kw).to(x.dtype)
    q = q.reshape(rows, heads, dim)
    f = 1 / torch.sqrt(k.float().pow(2).mean(1) + eps)
    k = k.reshape(rows, G, dim)
    out = torch.zeros(rows, heads, dim, dtype=x.dtype)
    sinks = None if sink is None else torch.full((heads,), float(sink))
    for r0, n, p0, s in _portions(plan):
        i = torch.arange(p0, p0 + n)
        cell = cache.table[s].long()[i // page]
        kc[cell, :, i % page] = k[r0:r0 + n]
        kf[cell, i % page] = f[r0:r0 + n]
        j = torch.arange(p0 - p0 % size if size else 0, p0 + n)
        cell = cache.table[s].long()[j // page]
        v = kc[cell, :, j % page]
        o = _attend(q[r0:r0 + n], v.float() * kf[cell, j % page].view(-1, 1, 1),
                    v, i, j, size=size, scale=scale, sink=sinks, slopes=slopes)
        if gated:
            o = o * torch.sigmoid(g[r0:r0 + n, :heads * dim].float()).view(
                n, heads, dim)
        out[r0:r0 + n] = o.to(x.dtype)
    return out.reshape(rows, heads * dim)


def retention(qkvg, cache, run, plan, *, pows, dec, rope, kscale, eps):
    """Retention of a ragged batch over run `run` of the cache's states.
    qkvg rows are [H*dk | H*dk | H*dv | H*dv]; rope: (cos, sin) tables of
    the rotated leading span, or None.  Returns (rows, H * dv): the
    normed, gated head outputs."""
    st, = cache.state[run]
    if qkvg.is_cuda:
        cos, sin = rope if rope is not None else (None, None)
        return require_lm_ext().retention(
            qkvg, st, plan.pos, plan.slot, plan.tiles, plan.seqs, plan.n_dec,
            pows, dec, cos, sin, kscale, eps, False)
    H, dv, dk = st.shape[1:]
    q, k, v, g = (t.reshape(qkvg.shape[0], H, -1).float() for t in
                  torch.split(qkvg, [H * dk, H * dk, H * dv, H * dv], dim=1))
    if rope is not None:
        c, s = (t[plan.pos.long()].unsqueeze(1) for t in rope)
        hf = c.shape[-1]

        def turn(x):
            u, w = x[..., :hf], x[..., hf:2 * hf]
            return torch.cat([u * c - w * s, w * c + u * s, x[..., 2 * hf:]], -1)

        q, k = turn(q), turn(k)
    k = k * kscale
    d = dec.sum(1).view(H, 1, 1)
    o = torch.zeros(qkvg.shape[0], H, dv)
    for r0, n, p0, sl in _portions(plan):
        S = torch.zeros_like(st[sl]) if p0 == 0 else st[sl]
        for r in range(r0, r0 + n):
            S = d * S + v[r].unsqueeze(2) * k[r].unsqueeze(1)
            o[r] = (S @ q[r].unsqueeze(2)).squeeze(2)
        st[sl] = S
    y = _rms(o, eps) * F.silu(g)
    return y.reshape(qkvg.shape[0], H * dv).to(qkvg.dtype)


def lightning(p, cache, run, plan, *, pows, dec, norm, eps):
    """Linear attention with a fixed decay per head over run `run` of the
    cache's states; rows of p are [q | k | v | gate], the first three through
    silu.  Returns (rows, H * dv): all heads together through an RMS norm with
    weights `norm`, times the gate's sigmoid."""
    st, = cache.state[run]
    if p.is_cuda:
        m = require_lm_ext()
        o = m.retention(p, st, plan.pos, plan.slot, plan.tiles, plan.seqs,
                        plan.n_dec, pows, dec, None, None, 1.0, eps, True)
        H, dv, dk = st.shape[1:]
        return m.gated_rms(o, norm, p, H * (2 * dk + dv), eps)
    H, dv, dk = st.shape[1:]
    q, k, v, g = torch.split(p.float(), [H * dk, H * dk, H * dv, H * dv], dim=1)
    q, k, v = (F.silu(t).view(p.shape[0], H, -1) for t in (q, k, v))
    d = dec.sum(1).view(H, 1, 1)
    o = torch.zeros(p.shape[0], H, dv)
    for r0, n, p0, sl in _portions(plan):
        S = torch.zeros_like(st[sl]) if p0 == 0 else st[sl]
        for r in range(r0, r0 + n):
            S = d * S + v[r].unsqueeze(2) * k[r].unsqueeze(1)
            o[r] = (S @ q[r].unsqueeze(2)).squeeze(2)
        st[sl] = S
    o = o.reshape(p.shape[0], H * dv).to(p.dtype)
    return (_rms(o, eps, norm) * torch.sigmoid(g)).to(p.dtype)


def gla(x, col, out, out_col, cache, run, plan, *, rank, a2, a2_b, tau, norm,
        out_scale, eps):
    """Gated linear attention (Yang et al., "Gated Linear Attention
    Transformers with Hardware-Efficient Training") of a ragged batch over run
    `run` of the cache's states: S <- diag(alpha) S + k v^T, o = S^T q /
    sqrt(dim), with alpha = sigmoid(a2 u + a2_b)^(1/tau) per key channel.  x's
    columns from `col` on are [q | k | v | gate | u], u `rank` wide.  Each
    head's result, RMS-normed (weights `norm`), times silu of its gate and
    out_scale, goes to out's columns from out_col on."""
    st = cache.state[run][0]
    if x.is_cuda:
        return require_lm_ext().gla(
            x, col, out, out_col, st, plan.pos, plan.slot, plan.tiles,
            plan.seqs, plan.n_dec, a2, a2_b, tau, norm, out_scale, eps)
    H, dv, dk = st.shape[1:]
    T = x.shape[0]
    q, k, v, g, u = torch.split(
        x[:, col:col + 2 * H * (dk + dv) + rank].float(),
        [H * dk, H * dk, H * dv, H * dv, rank], dim=1)
    alpha = torch.exp(F.logsigmoid(F.linear(u, a2.float(), a2_b.float())) / tau)
    q, k, v = (t.reshape(T, H, -1) for t in (q * dk ** -0.5, k, v))
    alpha = alpha.view(T, H, 1, dk)
    o = torch.zeros(T, H, dv)
    for r0, n, p0, s in _portions(plan):
        S = torch.zeros_like(st[s]) if p0 == 0 else st[s]
        for r in range(r0, r0 + n):
            S = alpha[r] * S + v[r].unsqueeze(2) * k[r].unsqueeze(1)
            o[r] = (S @ q[r].unsqueeze(2)).squeeze(2)
        st[s] = S
    y = _rms(o, eps, norm).reshape(T, H * dv) * F.silu(g) * out_scale
    out[:, out_col:out_col + H * dv] = y.to(x.dtype)


def latent_attention(a, cache, run, plan, *, heads, dim, vdim, rot, q_norm,
                     kv_norm, wuq, wuk, wuv, rope, size, scale, eps):
    """Latent attention of a ragged batch; appends its latents and rotated
    key parts to run `run` of the cache.  Rows of `a` are [query latent |
    key latent | shared key part | a gate per head]; wuq (heads*(dim+rot),
    q_rank), wuk (rank, heads*dim), wuv (heads*vdim, rank); rope: (cos,
    sin) of the rotated pairs or None; size: sliding window, 0 for plain
    causal.  Returns (rows, heads * vdim), gated.

    Prompt portions make keys and values of all the tokens they see from
    the latents; single tokens meet the latents themselves, the key matrix
    moved to the query's side and the value matrix behind the softmax."""
    q_rank, rank = q_norm.numel(), kv_norm.numel()
    kc = cache.k[run]
    if a.is_cuda:
        m = require_lm_ext()
        cos, sin = rope if rope is not None else (None, None)
        keys, blocks = (plan.spans(size) if plan.portions
                        else (plan.tiles, plan.tiles))
        cq, c, kr = m.latent_prep(a, kc, cache.table, plan.pos, plan.slot,
                                  keys, plan.n_dec, q_norm, kv_norm, rot, cos,
                                  sin, eps)
        q = linear(cq, wuq)
        k = v = None
        if plan.portions:
            k, v = c @ wuk, linear(c, wuv)
        return m.latent_attend(q, k, v, kr, a, kc, cache.table, plan.pos,
                               plan.slot, blocks, plan.n_dec, wuk, wuv, cos,
                               sin, heads, dim, vdim, rot, q_rank, size,
                               scale, cache.max_len)
    page = kc.shape[1]
    roff = -(-rank // 8) * 8           # where the key part starts in a row

    def turn(x, pos):                  # pairs (2i, 2i+1) of the last axis
        if rope is None:
            return x
        n = 2 * rope[0].shape[1]
        shape = (len(pos),) + (1,) * (x.dim() - 2) + (n // 2,)
        c, s = (t[pos].view(shape) for t in rope)
        u, w = x[..., 0:n:2], x[..., 1:n:2]
        y = torch.stack([u * c - w * s, w * c + u * s], -1).flatten(-2)
        return torch.cat([y, x[..., n:]], -1)

    dt = a.dtype
    cq = _rms(a[:, :q_rank], eps, q_norm).to(dt)
    c = _rms(a[:, q_rank:q_rank + rank], eps, kv_norm).to(dt)
    pos = plan.pos.long()
    kr = turn(a[:, q_rank + rank:q_rank + rank + rot].float(), pos).to(dt)
    gate = torch.sigmoid(a[:, q_rank + rank + rot:][:, :heads].float())
    q = (cq.float() @ wuq.float().T).to(dt).view(-1, heads, dim + rot).float()
    q = torch.cat([q[..., :dim], turn(q[..., dim:], pos)], -1)
    out = torch.zeros(a.shape[0], heads, vdim, dtype=dt)
    for r0, n, p0, s in _portions(plan):
        i = torch.arange(p0, p0 + n)
        cell = cache.table[s].long()[i // page]
        kc[cell, i % page, :rank] = c[r0:r0 + n]
        kc[cell, i % page, roff:roff + rot] = kr[r0:r0 + n]
        j = torch.arange(max(0, p0 - size + 1) if size else 0, p0 + n)
        row = kc[cache.table[s].long()[j // page], j % page]
        lat = row[:, :rank].float()
        ku = (lat @ wuk.float()).to(dt).float().view(-1, heads, dim)
        v = (lat @ wuv.float().T).to(dt).float().view(-1, heads, vdim)
        sc = (torch.einsum("ihd,jhd->hij", q[r0:r0 + n, :, :dim], ku)
              + torch.einsum("ihd,jd->hij", q[r0:r0 + n, :, dim:],
                             row[:, roff:roff + rot].float())) * scale
        see = j[None] <= i[:, None]
        if size:
            see &= i[:, None] - j[None] < size
        p = torch.softmax(sc.masked_fill(~see, float("-inf")), dim=2)
        o = torch.einsum("hij,jhe->ihe", p, v)
        out[r0:r0 + n] = (o * gate[r0:r0 + n].unsqueeze(2)).to(dt)
    return out.reshape(a.shape[0], heads * vdim)


def mamba2(p, cache, run, plan, *, groups, conv, conv_b, dt_bias, a_log,
           skip, norm, parts, eps):
    """State-space recurrence of a ragged batch over run `run` of the
    cache's states.  Rows of p are [z | x | B | C | step sizes]; returns
    (rows, inner), gated and normed."""
    st, tail = cache.state[run]
    H, dv, n = st.shape[1:]
    inner, taps = H * dv, conv.shape[1]
    if p.is_cuda:
        m = require_lm_ext()
        xbc = m.causal_conv(p, inner, conv, conv_b, tail, plan.pos, plan.slot,
                            plan.tiles, plan.seqs, plan.n_dec)
        y = m.mamba2(p, xbc, st, plan.pos, plan.slot, plan.tiles, plan.seqs,
                     plan.n_dec, groups, dt_bias, a_log, skip)
        return m.grouped_rms(y, norm, parts, eps)
    ch = conv.shape[0]
    z, xin = p[:, :inner].float(), p[:, inner:inner + ch].float()
    dt = F.softplus(p[:, inner + ch:][:, :H].float() + dt_bias.float(),
                    threshold=100.0)
    decay = torch.exp(-torch.exp(a_log.float()) * dt)
    y = torch.zeros(p.shape[0], H, dv)
    for r0, rows, p0, s in _portions(plan):
        past = torch.zeros_like(tail[s]) if p0 == 0 else tail[s]
        seq = torch.cat([past, xin[r0:r0 + rows]])
        u = conv_b.float() + sum(seq[a:a + rows] * conv[:, a].float()
                                 for a in range(taps))
        tail[s] = seq[rows:]
        x, B, C = torch.split(F.silu(u).to(p.dtype).float(),
                              [inner, groups * n, groups * n], dim=1)
        x = x.view(rows, H, dv)
        B, C = (t.view(rows, groups, n).repeat_interleave(H // groups, 1)
                for t in (B, C))
        S = torch.zeros_like(st[s]) if p0 == 0 else st[s]
        for r in range(rows):
            S = (decay[r0 + r].view(H, 1, 1) * S + dt[r0 + r].view(H, 1, 1)
                 * x[r].unsqueeze(2) * B[r].unsqueeze(1))
            y[r0 + r] = (S @ C[r].unsqueeze(2)).squeeze(2)
        y[r0:r0 + rows] += skip.float().view(H, 1) * x
        st[s] = S
    y = (y.reshape(-1, inner) * F.silu(z)).to(p.dtype)
    y = _rms(y.view(-1, parts, inner // parts), eps).reshape(-1, inner)
    return (y * norm.float()).to(p.dtype)


def mlstm(p, cache, run, plan, *, i_b, f_b, cap, norm, eps):
    """Matrix memory of a ragged batch over run `run` of the cache's
    states.  Rows of p are [q | k | v | output gate | input gate | forget
    gate]; returns (rows, heads * vdim), normed and gated."""
    st, sn, sm = cache.state[run]
    H, dv, dk = st.shape[1:]
    if p.is_cuda:
        return require_lm_ext().mlstm(
            p, st, sn, sm, plan.pos, plan.slot, plan.tiles, plan.seqs,
            plan.n_dec, i_b, f_b, cap, norm, eps)
    a, b = H * dk, H * dv
    q, k, v, g, i, f, _ = torch.split(
        p.float(), [a, a, b, b, H, H, p.shape[1] - 2 * (a + b + H)], dim=1)
    q = q.view(-1, H, dk) * dk ** -0.5
    k, v = k.view(-1, H, dk), v.view(-1, H, dv)
    i = cap * torch.tanh((i + i_b.float()) / cap)
    f = F.logsigmoid(cap * torch.tanh((f + f_b.float()) / cap))
    o = torch.zeros(p.shape[0], H, dv)
    for r0, rows, p0, s in _portions(plan):
        S, n, m = ((torch.zeros_like(t[s]) if p0 == 0 else t[s])
                   for t in (st, sn, sm))
        for r in range(r0, r0 + rows):
            top = torch.maximum(f[r] + m, i[r])
            keep, take = torch.exp(f[r] + m - top), torch.exp(i[r] - top)
            S = (keep.view(H, 1, 1) * S + take.view(H, 1, 1)
                 * v[r].unsqueeze(2) * k[r].unsqueeze(1))
            n = keep.view(H, 1) * n + take.view(H, 1) * k[r]
            m = top
            den = torch.maximum((n * q[r]).sum(1).abs(), torch.exp(-m))
            o[r] = (S @ q[r].unsqueeze(2)).squeeze(2) / (den.view(H, 1) + 1e-6)
        st[s], sn[s], sm[s] = S, n, m
    y = _rms(o, eps).reshape(-1, b) * norm.float() * torch.sigmoid(g)
    return y.to(p.dtype)


def moe(h, router, gate_up, down, shared, *, top, groups, keep, scale) -> Parts:
    """Routed gated experts of rows h (T, W).  router (rows, W): a logit per
    expert and, with a shared expert, the logit of its gate after them;
    gate_up (E, 2 ff, W), down (E, W, ff); shared: (gate_up, down) of an
    expert that every token takes, or None.  The experts are `groups` equal
    groups of neighbours; a token chooses its `top` best out of the `keep`
    groups whose two best scores have the largest sums.  Scores are
    sigmoids, an expert's weight is its score times `scale`."""
    if (h.is_cuda and h.dtype == torch.bfloat16 and h.shape[0] <= 64
            and h.shape[1] % 8 == 0):
        z = require_lm_ext().router_logits(h, router)
    else:
        z = linear_f32(h, router)
    if h.is_cuda:
        return Parts(*require_lm_ext().moe(h, z, gate_up, down,
                                           *(shared or (None, None)), top,
                                           groups, keep, scale))
    E, T = gate_up.shape[0], h.shape[0]
    s = torch.sigmoid(z[:, :E])
    per = s.view(T, groups, E // groups)
    merit = per.topk(min(2, E // groups), dim=2).values.sum(2)
    off = torch.ones(T, groups, dtype=torch.bool)
    off.scatter_(1, merit.topk(keep, dim=1).indices, False)
    ids = z[:, :E].masked_fill(off.repeat_interleave(E // groups, 1),
                               float("-inf")).topk(top, dim=1).indices
    weights = s.gather(1, ids) * scale
    y = _experts(h, ids, gate_up, down)
    if shared is not None:
        y = torch.cat([y, _expert(h, *shared).unsqueeze(1)], 1)
        weights = torch.cat([weights, torch.sigmoid(z[:, E:E + 1])], 1)
    return Parts(y, weights)


def table_moe(h, tokens, table, gate_up, down) -> Parts:
    """Gated experts of rows h (T, W), chosen by token id: table (vocab, top)
    int32 names each token's experts, which have equal weights; gate_up
    (E, 2 ff, W), down (E, W, ff)."""
    if h.is_cuda:
        return Parts(*require_lm_ext().table_moe(h, tokens, table, gate_up,
                                                 down))
    ids = table[tokens].long()
    return Parts(_experts(h, ids, gate_up, down),
                 torch.full(ids.shape, 1.0 / ids.shape[1]))


def _expert(x, gu, dn):
    g, u = F.linear(x.float(), gu.float()).to(x.dtype).float().chunk(2, -1)
    return F.linear((F.silu(g) * u).to(x.dtype).float(), dn.float()).to(x.dtype)


def _experts(h, ids, gate_up, down):
    """(T, top, W): every row by each of its experts ids (T, top)."""
    y = h.new_empty(*ids.shape, h.shape[1])
    for e in range(gate_up.shape[0]):
        t, k = (ids == e).nonzero(as_tuple=True)
        if t.numel():
            y[t, k] = _expert(h[t], gate_up[e], down[e])
    return y
