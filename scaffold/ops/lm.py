"""Ops of the mixer-stack models (paged attention, retention, residual
norms).  GPU tensors run the HIP kernels of csrc/lm, required; CPU tensors
run the plain float32 forms below, which the CPU tests use.
"""

from __future__ import annotations

from typing import Optional, Tuple

import torch
import torch.nn.functional as F

from .backend import require_lm_ext


def rope_tables_exact(seq_len: int, dims: int, base: float, device
                      ) -> Tuple[torch.Tensor, torch.Tensor]:
    """cos/sin (seq_len, dims/2) in float32, angles in float64: the table
    entries carry no error of the angle, however long the sequence."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    ang = torch.outer(torch.arange(seq_len, dtype=torch.float64),
                      float(base) ** (-2.0 * i / dims))
    return (ang.cos().float().to(device).contiguous(),
            ang.sin().float().to(device).contiguous())


def decay_tables(decay, tile: int, device) -> Tuple[torch.Tensor, torch.Tensor]:
    """(powers (H, tile+1) = decay^n, decays (H, 2) as float + remainder)."""
    d = torch.tensor(decay, dtype=torch.float64)
    n = torch.arange(tile + 1, dtype=torch.float64)
    pows = d.unsqueeze(1) ** n
    hi = d.float()
    lo = (d - hi.double()).float()
    return (pows.float().to(device).contiguous(),
            torch.stack([hi, lo], 1).to(device).contiguous())


def _ln(x, w, b, eps):
    return F.layer_norm(x.float(), (x.shape[-1],), w.float(),
                        None if b is None else b.float(), eps)


def embed_norm(tokens, embed, w, b, eps):
    """Residual stream x (float32) of the tokens and its first norm."""
    if embed.is_cuda:
        return require_lm_ext().embed_norm(tokens, embed, w, b, eps)
    x = embed[tokens].float()
    return x, _ln(x, w, b, eps).to(embed.dtype)


def residual_norm(x, y, post, mult, nxt, eps, rows=None, store_x=True):
    """x += mult * LN(y; post) (post None: y itself), then LN(x; nxt) of
    `rows` (None: all).  post and nxt are (weight, bias or None)."""
    pw, pb = post if post is not None else (None, None)
    if x.is_cuda:
        return require_lm_ext().residual_norm(
            x, y, pw, pb, mult, nxt[0], nxt[1], rows, eps, store_x)
    z = x
    if y is not None:
        z = x + mult * (y.float() if pw is None else _ln(y, pw, pb, eps))
        if store_x:
            x.copy_(z)
    if rows is not None:
        z = z[rows.long()]
    return _ln(z, nxt[0], nxt[1], eps).to(nxt[0].dtype)


def gelu_erf(x):
    if x.is_cuda:
        return require_lm_ext().gelu_erf(x)
    return F.gelu(x.float()).to(x.dtype)


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


def paged_attention(qkv, cache, run, plan, *, heads, q_norm, k_norm, sink,
                    size, scale, eps):
    """Attention of a ragged batch; appends its keys and values to run
    `run` of the cache.  qkv rows are [heads*dim | kv*dim | kv*vdim];
    q_norm, k_norm: per-head RMS weights or None; sink: (heads,) added to
    the softmax denominator, or None; size: chunk length, 0 for plain
    causal.  Returns (rows, heads * vdim)."""
    kc, vc = cache.k[run], cache.v[run]
    if qkv.is_cuda:
        return require_lm_ext().paged_attention(
            qkv, kc, vc, cache.table, plan.pos, plan.slot, plan.tiles,
            plan.n_dec, q_norm, k_norm, sink, heads, size, scale, eps,
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
        rep = heads // G
        kk = kc[cell, :, j % page].float().repeat_interleave(rep, 1)
        vv = vc[cell, :, j % page].float().repeat_interleave(rep, 1)
        sc = torch.einsum("ihd,jhd->hij", q[r0:r0 + n].float(), kk) * scale
        see = j[None] <= i[:, None]
        if size:
            see &= j[None] // size == i[:, None] // size
        sc = sc.masked_fill(~see, float("-inf"))
        if sink is not None:
            sc = torch.cat([sc, sink.float().view(-1, 1, 1).expand(-1, n, 1)], 2)
        p = torch.softmax(sc, dim=2)[:, :, :j.numel()]
        out[r0:r0 + n] = torch.einsum("hij,jhe->ihe", p, vv).to(qkv.dtype)
    return out.reshape(qkv.shape[0], heads * vdim)


def retention(qkvg, cache, run, plan, *, pows, dec, rope, kscale, eps):
    """Retention of a ragged batch over run `run` of the cache's states.
    qkvg rows are [H*dk | H*dk | H*dv | H*dv]; rope: (cos, sin) tables of
    the rotated leading span, or None.  Returns (rows, H * dv): the
    normed, gated head outputs."""
    st = cache.state[run]
    if qkvg.is_cuda:
        cos, sin = rope if rope is not None else (None, None)
        return require_lm_ext().retention(
            qkvg, st, plan.pos, plan.slot, plan.tiles, plan.seqs, plan.n_dec,
            pows, dec, cos, sin, kscale, eps)
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
