"""Mixer-stack language models: a decoder whose layers are listed one by
one, each with its own token mixer and an optional feed-forward, and a
span of which may run several times with the same weights.

The model owns weights and one function, `forward_step`, that runs a
ragged batch (StepPlan) over a PagedStateCache; scaffold.generate drives
it for generation, serving and trace replay.  Mixers and feed-forwards
come from scaffold.models.mixers.  The residual stream is float32
throughout.

What a configuration can choose besides the layers: the kind of norm,
whether sublayers have one before them, after them or both, learned or
sinusoidal position vectors, a vector per pair of neighbouring tokens, a
blend of every mixer's input with the previous token's, a factor of every
sublayer, what happens before each pass of the repeated span (a projection of
the stream and the embeddings, or the embeddings and a vector of the pass
added to the stream), and a soft cap on the logits.
"""

from __future__ import annotations

from typing import Callable, Dict, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..cache import PagedStateCache, StateSpec, StepPlan
from .gpt2 import LayerNorm
from .mixers import FEED_FORWARDS, MIXERS


class DynamicTanh(nn.Module):
    """tanh(alpha * x) * weight + bias, a norm without statistics."""

    def __init__(self, width: int, eps: float = 0.0):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(width))
        self.bias = nn.Parameter(torch.zeros(width))
        self.alpha = nn.Parameter(torch.tensor(0.5))


class RMSNorm(nn.Module):
    """x over its root mean square, times weight."""

    def __init__(self, width: int, eps: float):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(width))


class ScalarRMSNorm(nn.Module):
    """x over its root mean square, times one number."""

    def __init__(self, width: int, eps: float):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(()))


NORMS = {"layer_norm": LayerNorm, "rms_norm": RMSNorm,
         "scalar_rms_norm": ScalarRMSNorm, "dynamic_tanh": DynamicTanh}


def _lookup(table: dict, name: str, what: str):
    if name not in table:
        raise ValueError(f"unknown {what} {name!r} (known: "
                         f"{', '.join(sorted(table))})")
    return table[name]


class StackLayer(nn.Module):
    """One layer: (norm1 ->) (blend with the previous token's ->) mixer
    (-> norm1b), then (if it has one) (norm2 ->) feed-forward (-> norm2b)."""

    def __init__(self, m, spec: dict):
        super().__init__()
        width, eps = m.d_model, m.norm_eps
        norm = _lookup(NORMS, m.norm, "norm")
        ff = spec.get("mlp")
        for n in ("norm1", "norm2")[:1 if ff is None else 2]:
            setattr(self, n, norm(width, eps) if m.pre_norm else None)
            setattr(self, n + "b", norm(width, eps) if m.post_norm else None)
        self.shift = (nn.Parameter(torch.full((width,), 0.5))
                      if m.token_shift else None)
        self.mixer = _lookup(MIXERS, spec["type"], "mixer")(
            width, spec["mixer"], eps)
        self.ff = None
        if ff is not None:
            self.ff = _lookup(FEED_FORWARDS, ff["kind"], "feed-forward")(
                width, ff, m.vocab_size)


def _params(norm) -> Optional[tuple]:
    """A norm as the ops take it: (weight,) without a bias, (weight, bias),
    and alpha if it has one."""
    if norm is None:
        return None
    if not hasattr(norm, "bias"):
        return (norm.weight,)
    alpha = getattr(norm, "alpha", None)
    return (norm.weight, norm.bias) + (() if alpha is None else (alpha,))


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
        self.softcap = float(m.logit_softcap)
        self.vocab = m.vocab_size
        self.max_seq_len = m.max_seq_len
        self.embed = nn.Embedding(m.vocab_size, m.d_model)
        # learned position vectors; they end the longest sequence
        self.pos = None
        if m.positions:
            self.pos = nn.Embedding(m.positions, m.d_model)
            self.max_seq_len = min(m.max_seq_len, m.positions)
        # a vector per pair of neighbouring tokens, the last row for a
        # sequence's first token; turns per position of sinusoidal vectors
        self.bigram = None
        if m.bigram:
            self.pair_mul = m.bigram["mul_prev"], m.bigram["mul_cur"]
            self.bigram = nn.Embedding(m.bigram["buckets"] + 1, m.d_model)
        self.sinusoid_base = float(m.sinusoid_base)
        self._rates: Dict[str, torch.Tensor] = {}
        if m.positions and (self.bigram is not None or self.sinusoid_base):
            raise ValueError("learned positions beside sinusoids or pairs")
        # streams that make a mixer's input in shift_norm
        self.shifted = m.token_shift
        if (m.token_shift or m.loop_add) and (m.post_norm or not m.pre_norm
                                              or m.loop_input):
            raise ValueError("token_shift and loop_add go with pre_norm alone")
        self.blocks = nn.ModuleList(StackLayer(m, s) for s in m.layers)
        self.norm_f = _lookup(NORMS, m.norm, "norm")(m.d_model, m.norm_eps)
        self.lm_head = nn.Linear(m.d_model, m.vocab_size, bias=False)
        n = len(m.layers)
        loop = m.loop or {"start": 0, "stop": n, "times": 1}
        lo, hi, times = loop["start"], loop["stop"], loop["times"]
        if not 0 <= lo <= hi <= n or times < 1:
            raise ValueError(f"bad loop {loop} for {n} layers")
        # the layers in running order; position in this list = cache run
        self.runs: List[int] = [*range(lo), *([*range(lo, hi)] * times),
                                *range(hi, n)]
        # runs that begin a pass with something of their own (loop_input,
        # loop_add) -> the number of the pass
        self.entries: Dict[int, int] = {}
        self.loop_in = None
        if m.loop and (m.loop_input or m.loop_add):
            if lo == hi:
                raise ValueError(f"loop {loop} repeats no layer")
            self.entries = {lo + t * (hi - lo): t for t in range(times)}
            if m.loop_input:
                self.loop_in = nn.Linear(2 * m.d_model, m.d_model, bias=False)
            self.loop_step = nn.Parameter(torch.zeros(times, m.d_model))
        for p in self.parameters():
            if p.dim() > 1:
                nn.init.normal_(p, std=0.02)

    def named_views(self):
        """(checkpoint name, view of the weight) of every tensor."""
        def norm(name, mod):
            out = [(name, mod.weight)]
            if hasattr(mod, "bias"):
                out.append((name + ".b", mod.bias))
            if hasattr(mod, "alpha"):
                out.append((name + ".alpha", mod.alpha))
            return out

        out = [("embed", self.embed.weight)]
        if self.pos is not None:
            out.append(("pos", self.pos.weight))
        if self.bigram is not None:
            out.append(("bigram", self.bigram.weight))
        if self.loop_in is not None:
            out.append(("loop.in", self.loop_in.weight))
        if self.entries:
            out.append(("loop.step", self.loop_step))
        for i, blk in enumerate(self.blocks):
            for n in ("norm1", "norm1b", "norm2", "norm2b"):
                if getattr(blk, n, None) is not None:
                    # the only norm of a sublayer has the plain name
                    name = n if self.cfg.model.pre_norm else n.rstrip("b")
                    out += norm(f"l{i}.{name}", getattr(blk, n))
            out += [(f"l{i}.mix.{n}", t) for n, t in blk.mixer.packed()]
            if blk.ff is not None:
                out += [(f"l{i}.mlp.{n}", t) for n, t in blk.ff.packed()]
            if blk.shift is not None:
                out.append((f"l{i}.shift", blk.shift))
        return out + norm("final.norm", self.norm_f) + [
            ("head", self.lm_head.weight)]

    # ---- serving --------------------------------------------------------
    def new_cache(self, n_slots: int, n_tokens: int, max_len: int
                  ) -> PagedStateCache:
        w = self.embed.weight
        if self.pos is not None:
            max_len = min(max_len, self.pos.num_embeddings)
        specs = [self.blocks[i].mixer.cache_spec() for i in self.runs]
        # behind the layer runs: what their inputs look back at, then the
        # token before
        if self.shifted:
            specs += [StateSpec(((w.shape[1],),))] * len(self.runs)
        if self.bigram is not None:
            specs.append(StateSpec(((),), torch.int64))
        return PagedStateCache(specs, n_slots, n_tokens, max_len, w.device,
                               w.dtype)

    def _embed(self, plan: StepPlan, cache: PagedStateCache) -> torch.Tensor:
        """The stream as the embeddings leave it (sinusoids, pairs)."""
        w, rates = self.embed.weight, None
        if self.sinusoid_base:
            key = str(w.device)
            if key not in self._rates:
                self._rates[key] = ops.turn_rates(w.shape[1],
                                                  self.sinusoid_base, w.device)
            rates = self._rates[key]
        if self.bigram is None:
            return ops.stream_embed(plan, w, rates=rates)
        return ops.stream_embed(plan, w, rates=rates, pairs=self.bigram.weight,
                                mul=self.pair_mul, last=cache.state[-1][0])

    def _logits(self, h: torch.Tensor) -> torch.Tensor:
        if not self.softcap:
            return ops.linear(h, self.lm_head.weight)
        return ops.softcap(ops.linear_f32(h, self.lm_head.weight),
                           self.softcap)

    @torch.no_grad()
    def forward_step(self, plan: StepPlan, cache: PagedStateCache,
                     on_layer: Optional[Callable] = None) -> torch.Tensor:
        """Run the plan's tokens and return the logits of its wanted rows
        (rows, vocab).  Keys, values and states go into the cache.
        on_layer(run, x) sees the residual stream after every layer run."""
        blocks, eps, embed = self.blocks, self.eps, self.embed.weight
        last = len(self.runs) - 1
        rows = plan.rows
        own_start = bool(self.sinusoid_base) or self.bigram is not None
        added = bool(self.entries) and self.loop_in is None

        def first(run):
            return _params(blocks[self.runs[run]].norm1)

        def begin_pass(run, x, y, post):
            """Project stream and embeddings, and norm for the first layer."""
            both = ops.residual_concat(x, y, post, self.mult, eps,
                                       plan.tokens, embed)
            if on_layer is not None and run:
                on_layer(run - 1, x)
            return x, ops.replace_norm(
                x, ops.linear_f32(both, self.loop_in.weight),
                self.loop_step[self.entries[run]], first(run), eps)

        def mixer_input(run, x, y):
            """The stream with y added, what begins a pass included, and
            run's input."""
            blk, n = blocks[self.runs[run]], self.entries.get(run)
            if on_layer is not None and run:
                x, _ = ops.shift_norm(x, y, self.mult, first(run), eps, plan)
                on_layer(run - 1, x)
                y = None
            state = cache.state[last + 1 + run][0] if self.shifted else None
            return ops.shift_norm(
                x, y, self.mult, first(run), eps, plan, shift=blk.shift,
                state=state, add=start if n else None,
                step=None if n is None else self.loop_step[n])

        if own_start:
            start = x = self._embed(plan, cache)
            if not (self.shifted or added):
                h = ops.residual_norm(x, None, None, 1.0, first(0), eps)
        else:
            x, h = ops.embed_norm(plan.tokens, embed, first(0), eps, plan.pos,
                                  None if self.pos is None else self.pos.weight)
            start = x
        if self.shifted or added:
            x, h = mixer_input(0, x, None)
        elif 0 in self.entries:
            x, h = begin_pass(0, x, None, None)
        for run, i in enumerate(self.runs):
            blk = blocks[i]
            end = run == last
            y, post = blk.mixer.step(h, plan, cache, run), blk.norm1b
            if (end and rows is not None and rows.numel() == 0
                    and on_layer is None):
                # nothing wanted, and the last run's cache is filled
                return self._logits(h.new_zeros(0, h.shape[1]))
            if blk.ff is not None:
                h = ops.residual_norm(x, y, _params(post), self.mult,
                                      _params(blk.norm2), eps)
                y, post = blk.ff.step(h, plan), blk.norm2b
            if not end and (self.shifted or added):
                x, h = mixer_input(run + 1, x, y)
                continue
            if run + 1 in self.entries:
                x, h = begin_pass(run + 1, x, y, _params(post))
                continue
            # only wanted rows pass the last norm, unless someone watches x
            few = end and rows is not None and on_layer is None
            h = ops.residual_norm(
                x, y, _params(post), self.mult,
                _params(self.norm_f) if end else first(run + 1), eps,
                rows=rows if few else None, store_x=not few)
            if on_layer is not None:
                on_layer(run, x)
        if rows is not None and on_layer is not None:
            h = h[rows.long()]
        return self._logits(h)

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
