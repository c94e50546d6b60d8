"""Mixer-stack language models: a decoder whose layers are listed one by
one, each with its own token mixer and an optional feed-forward, and a
span of which may run several times with the same weights.

The model owns weights and one function, `forward_step`, that runs a
ragged batch (StepPlan) over a PagedStateCache; scaffold.generate drives
it for generation, serving and trace replay.  Mixers are looked up by
name in MIXERS; each states what it caches (cache_spec) and computes its
part of a step (step).  The residual stream is float32 throughout.

Lasezen is the design built from: layer norms before and after every
sublayer, chunk-local attention with normed queries and keys and a
learned sink, retention with a constant decay per head, exact-GELU
feed-forwards.
"""

from __future__ import annotations

from typing import Callable, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..cache import TILE, KVSpec, PagedStateCache, StateSpec, StepPlan
from .gpt2 import LayerNorm


class ChunkAttention(nn.Module):
    """Grouped-query attention inside consecutive chunks of mask.size
    tokens (absent: plain causal), with per-head RMS norms on queries and
    keys and a learned sink per head."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.kv = spec["heads"], spec["kv_heads"]
        self.dim, self.vdim = spec["dim"], spec["vdim"]
        self.scale = float(spec["scale"])
        self.size = int((spec.get("mask") or {}).get("size", 0))
        self.eps = eps
        if self.heads % self.kv:
            raise ValueError(f"kv_heads {self.kv} must divide heads "
                             f"{self.heads}")
        self.wqkv = nn.Linear(width, (self.heads + self.kv) * self.dim
                              + self.kv * self.vdim, bias=False)
        self.q_norm = nn.Parameter(torch.ones(self.dim))
        self.k_norm = nn.Parameter(torch.ones(self.dim))
        self.sink = nn.Parameter(torch.zeros(self.heads))
        self.wo = nn.Linear(self.heads * self.vdim, width, bias=False)

    def packed(self):
        """(checkpoint name, module weight, first row, rows)."""
        q, k, v = (self.heads * self.dim, self.kv * self.dim,
                   self.kv * self.vdim)
        w = self.wqkv.weight
        return [("q", w, 0, q), ("k", w, q, k), ("v", w, q + k, v),
                ("q.norm", self.q_norm, 0, self.dim),
                ("k.norm", self.k_norm, 0, self.dim),
                ("sink", self.sink, 0, self.heads),
                ("o", self.wo.weight, 0, self.wo.weight.shape[0])]

    def cache_spec(self):
        return KVSpec(self.kv, self.dim, self.vdim)

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        o = ops.paged_attention(
            ops.linear(h, self.wqkv.weight), cache, run, plan,
            heads=self.heads, q_norm=self.q_norm, k_norm=self.k_norm,
            sink=self.sink, size=self.size, scale=self.scale, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class Retention(nn.Module):
    """Linear attention with a fixed decay per head, rotated queries and
    keys, a per-head output norm and a silu gate."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.dim, self.vdim = (spec["heads"], spec["dim"],
                                           spec["vdim"])
        self.decay = [float(d) for d in spec["decay"]]
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} "
                             "heads")
        rot = spec.get("rot") or {}
        self.rot_dims = int(rot.get("dims", 0))
        self.rot_base = float(rot.get("base", 1.0))
        if self.rot_dims % 2 or self.rot_dims > self.dim:
            raise ValueError(f"rot.dims {self.rot_dims} must be even and at "
                             f"most dim {self.dim}")
        self.eps = eps
        self.wqkvg = nn.Linear(width, 2 * self.heads * (self.dim + self.vdim),
                               bias=False)
        self.wo = nn.Linear(self.heads * self.vdim, width, bias=False)
        self._tables = {}      # device -> decay tables (always float32)

    def packed(self):
        a, b = self.heads * self.dim, self.heads * self.vdim
        w = self.wqkvg.weight
        return [("q", w, 0, a), ("k", w, a, a), ("v", w, 2 * a, b),
                ("g", w, 2 * a + b, b),
                ("o", self.wo.weight, 0, self.wo.weight.shape[0])]

    def cache_spec(self):
        return StateSpec(self.heads, self.dim, self.vdim)

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        key = str(h.device)
        if key not in self._tables:
            self._tables[key] = ops.decay_tables(self.decay, TILE, h.device)
        pows, dec = self._tables[key]
        rope = (cache.rope(self.rot_base, self.rot_dims)
                if self.rot_dims else None)
        o = ops.retention(ops.linear(h, self.wqkvg.weight), cache, run, plan,
                          pows=pows, dec=dec, rope=rope,
                          kscale=self.dim ** -0.5, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class DenseFF(nn.Module):
    def __init__(self, width: int, spec: dict):
        super().__init__()
        self.up = nn.Linear(width, spec["ff"], bias=False)
        self.down = nn.Linear(spec["ff"], width, bias=False)

    def packed(self):
        return [("up", self.up.weight, 0, self.up.weight.shape[0]),
                ("down", self.down.weight, 0, self.down.weight.shape[0])]

    def step(self, h):
        return ops.linear(ops.gelu_erf(ops.linear(h, self.up.weight)),
                          self.down.weight)


MIXERS = {"attention": ChunkAttention, "retention": Retention}
FEED_FORWARDS = {"dense": DenseFF}


def _lookup(table: dict, name: str, what: str):
    if name not in table:
        raise ValueError(f"unknown {what} {name!r} (known: "
                         f"{', '.join(sorted(table))})")
    return table[name]


class StackLayer(nn.Module):
    """One layer: norm1 -> mixer -> norm1b, then (if it has one)
    norm2 -> feed-forward -> norm2b."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.norm1 = LayerNorm(width, eps)
        self.norm1b = LayerNorm(width, eps)
        self.mixer = _lookup(MIXERS, spec["type"], "mixer")(
            width, spec["mixer"], eps)
        ff = spec.get("mlp")
        self.ff = None
        if ff is not None:
            self.norm2 = LayerNorm(width, eps)
            self.norm2b = LayerNorm(width, eps)
            self.ff = _lookup(FEED_FORWARDS, ff["kind"], "feed-forward")(
                width, ff)


def _wb(norm: LayerNorm):
    return norm.weight, norm.bias


class MixerStack(nn.Module):
    def __init__(self, cfg):
        super().__init__()
        m = cfg.model
        if not m.layers:
            raise ValueError("model.layers is empty: give the layer list "
                             "(or model.dir, a folder with config.json)")
        self.cfg = cfg
        self.eps = m.norm_eps
        self.mult = float(m.residual_mult)
        self.vocab = m.vocab_size
        self.max_seq_len = m.max_seq_len
        self.embed = nn.Embedding(m.vocab_size, m.d_model)
        self.blocks = nn.ModuleList(StackLayer(m.d_model, s, m.norm_eps)
                                    for s in m.layers)
        self.norm_f = LayerNorm(m.d_model, m.norm_eps)
        self.lm_head = nn.Linear(m.d_model, m.vocab_size, bias=False)
        n = len(m.layers)
        loop = m.loop or {"start": 0, "stop": n, "times": 1}
        lo, hi, times = loop["start"], loop["stop"], loop["times"]
        if not 0 <= lo <= hi <= n or times < 1:
            raise ValueError(f"bad loop {loop} for {n} layers")
        # the layers in running order; position in this list = cache run
        self.runs: List[int] = [*range(lo), *([*range(lo, hi)] * times),
                                *range(hi, n)]
        for p in self.parameters():
            if p.dim() > 1:
                nn.init.normal_(p, std=0.02)

    # ---- serving --------------------------------------------------------
    def new_cache(self, n_slots: int, n_tokens: int, max_len: int
                  ) -> PagedStateCache:
        w = self.embed.weight
        return PagedStateCache([self.blocks[i].mixer.cache_spec()
                                for i in self.runs], n_slots, n_tokens,
                               max_len, w.device, w.dtype)

    @torch.no_grad()
    def forward_step(self, plan: StepPlan, cache: PagedStateCache,
                     on_layer: Optional[Callable] = None) -> torch.Tensor:
        """Run the plan's tokens and return the logits of its wanted rows
        (rows, vocab).  Keys, values and states go into the cache.
        on_layer(run, x) sees the residual stream after every layer run."""
        blocks, eps = self.blocks, self.eps
        x, h = ops.embed_norm(plan.tokens, self.embed.weight,
                              *_wb(blocks[self.runs[0]].norm1), eps)
        last = len(self.runs) - 1
        rows = plan.rows
        for run, i in enumerate(self.runs):
            blk = blocks[i]
            end = run == last
            # the norm that reads the stream after this layer
            nxt = self.norm_f if end else blocks[self.runs[run + 1]].norm1
            y, post = blk.mixer.step(h, plan, cache, run), blk.norm1b
            if (end and rows is not None and rows.numel() == 0
                    and on_layer is None):
                # nothing wanted, and the last run's cache is filled
                return h.new_zeros(0, self.vocab)
            if blk.ff is not None:
                h = ops.residual_norm(x, y, _wb(post), self.mult,
                                      _wb(blk.norm2), eps)
                y, post = blk.ff.step(h), blk.norm2b
            # only wanted rows pass the last norm, unless someone watches x
            few = end and rows is not None and on_layer is None
            h = ops.residual_norm(x, y, _wb(post), self.mult, _wb(nxt), eps,
                                  rows=rows if few else None,
                                  store_x=not few)
            if on_layer is not None:
                on_layer(run, x)
        if rows is not None and on_layer is not None:
            h = h[rows.long()]
        return ops.linear(h, self.lm_head.weight)

    # ---- scoring --------------------------------------------------------
    def forward(self, tokens: torch.Tensor, targets: torch.Tensor
                ) -> torch.Tensor:
        """Mean cross-entropy of (B, S) tokens against targets, through
        the serving step.  Inference only: the kernels have no backward."""
        if torch.is_grad_enabled() and self.training:
            raise NotImplementedError(
                "mixer-stack models have no backward; score them in eval "
                "mode or under torch.no_grad()")
        B, S = tokens.shape
        cache = self.new_cache(B, B * (-(-S // 64) * 64), S)
        entries = [(cache.open(), tokens[b], range(S)) for b in range(B)]
        plan, _ = cache.plan(entries)
        logits = self.forward_step(plan, cache)
        return torch.nn.functional.cross_entropy(logits.float(),
                                                 targets.reshape(-1))
