"""Token mixers and feed-forwards of mixer-stack models.

Each mixer states what it caches (cache_spec), computes its part of a step
(step) and names its weights as checkpoints do (packed); projections that
share an input are one matrix here and separate tensors there.  MIXERS and
FEED_FORWARDS look them up by name.
"""

from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from ..cache import (TILE, KVSpec, LatentSpec, PagedStateCache, StateSpec,
                     StepPlan, TiedSpec)


def _cut(w: torch.Tensor, **rows: int):
    """(name, row span) pairs of a packed weight, in order."""
    out, at = [], 0
    for name, n in rows.items():
        out.append((name, w[at:at + n]))
        at += n
    return out


def _pad8(n: int) -> int:
    """Packed rows are padded so that every row of a product starts 16
    bytes aligned; the extra outputs are not read."""
    return -(-n // 8) * 8


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
        return _cut(self.wqkv.weight, q=self.heads * self.dim,
                    k=self.kv * self.dim, v=self.kv * self.vdim) + [
            ("q.norm", self.q_norm), ("k.norm", self.k_norm),
            ("sink", self.sink), ("o", self.wo.weight)]

    def cache_spec(self):
        return KVSpec(self.kv, self.dim, self.vdim)

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        o = ops.paged_attention(
            ops.linear(h, self.wqkv.weight), cache, run, plan,
            heads=self.heads, q_norm=self.q_norm, k_norm=self.k_norm,
            sink=self.sink, size=self.size, scale=self.scale, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class TiedAttention(nn.Module):
    """Grouped-query attention whose values are its keys (before their
    norm), with biases on both projections, RMS norms over all heads at
    once, a query temperature that grows with the position, scores that
    lose a fixed slope per step of distance (the geometric slopes of Press
    et al., "Train Short, Test Long: Attention with Linear Biases Enables
    Input Length Extrapolation"), a constant sink and a gate per element."""

    SINK = 0.0     # exp of it is added to the softmax denominator

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.kv, self.dim = (spec["heads"], spec["kv_heads"],
                                         spec["dim"])
        self.scale = float(spec["scale"])
        self.size = int((spec.get("mask") or {}).get("size") or 0)
        temp = spec.get("q_temp")
        self.temp = temp and (float(temp["coef"]), int(temp["every"]))
        self.eps = eps
        if self.heads % self.kv:
            raise ValueError(f"kv_heads {self.kv} must divide heads "
                             f"{self.heads}")
        if spec.get("vdim", self.dim) != self.dim:
            raise ValueError(f"vdim {spec['vdim']}: values are keys, of dim "
                             f"{self.dim}")
        if self.temp and self.temp[1] < 1:
            raise ValueError(f"q_temp.every {self.temp[1]} must be positive")
        # rows: q | k | gate
        a, b = self.heads * self.dim, self.kv * self.dim
        self.win = nn.Linear(width, _pad8(2 * a + b))
        nn.init.zeros_(self.win.bias)
        self.q_norm = nn.Parameter(torch.ones(a))
        self.k_norm = nn.Parameter(torch.ones(b))
        self.wo = nn.Linear(a, width, bias=False)
        self._slopes = {}      # device -> slopes (always float32)

    def packed(self):
        a, b = self.heads * self.dim, self.kv * self.dim
        return (_cut(self.win.weight, q=a, k=b, g=a)
                + _cut(self.win.bias, **{"q.b": a, "k.b": b})
                + [("q.norm", self.q_norm), ("k.norm", self.k_norm),
                   ("o", self.wo.weight)])

    def cache_spec(self):
        return TiedSpec(self.kv, self.dim)

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        key = str(h.device)
        if key not in self._slopes:
            self._slopes[key] = torch.tensor(
                [2.0 ** (-8.0 * (i + 1) / self.heads)
                 for i in range(self.heads)], device=h.device)
        o = ops.tied_attention(
            ops.linear(h, self.win.weight, self.win.bias), cache, run, plan,
            heads=self.heads, q_norm=self.q_norm, k_norm=self.k_norm,
            temp=self.temp, slopes=self._slopes[key], sink=self.SINK,
            gated=True, size=self.size, scale=self.scale, eps=self.eps)
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
        return (_cut(self.wqkvg.weight, q=a, k=a, v=b, g=b)
                + [("o", self.wo.weight)])

    def cache_spec(self):
        # transposed, [vdim][dim]: the order the kernels read
        return StateSpec(((self.heads, self.vdim, self.dim),))

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


class LatentAttention(nn.Module):
    """Attention whose keys and values are made from a cached latent, with
    one rotated key part shared by all heads, queries through a latent of
    their own, a sliding window of mask.size tokens (absent: plain causal)
    and a sigmoid gate per head.  rot.scaling: YaRN's constants."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.dim, self.vdim = (spec["heads"], spec["dim"],
                                           spec["vdim"])
        self.rot, self.rank, self.q_rank = (spec["rot_dim"], spec["kv_rank"],
                                            spec["q_rank"])
        self.scale = float(spec["scale"])
        self.size = int((spec.get("mask") or {}).get("size") or 0)
        rot = spec.get("rot") or {}
        self.rot_dims = int(rot.get("dims", 0))
        self.rot_base = float(rot.get("base", 1.0))
        self.rot_scaling = rot.get("scaling")
        if self.rot_dims % 2 or self.rot_dims > self.rot:
            raise ValueError(f"rot.dims {self.rot_dims} must be even and at "
                             f"most rot_dim {self.rot}")
        self.eps = eps
        # rows: query latent | key latent, shared key part | head gates
        self.win = nn.Linear(width, _pad8(self.q_rank + self.rank + self.rot
                                          + self.heads), bias=False)
        self.q_norm = nn.Parameter(torch.ones(self.q_rank))
        self.kv_norm = nn.Parameter(torch.ones(self.rank))
        self.wuq = nn.Linear(self.q_rank, self.heads * (self.dim + self.rot),
                             bias=False)
        # latent -> keys, kept [rank, heads*dim]: prompts multiply by it,
        # decoding by its transpose, both along rows
        self.wuk = nn.Parameter(torch.empty(self.rank, self.heads * self.dim))
        self.wuv = nn.Linear(self.rank, self.heads * self.vdim, bias=False)
        self.wo = nn.Linear(self.heads * self.vdim, width, bias=False)

    def packed(self):
        return _cut(self.win.weight, dq=self.q_rank, dkv=self.rank + self.rot,
                    g=self.heads) + [
            ("dq.norm", self.q_norm), ("dkv.norm", self.kv_norm),
            ("uq", self.wuq.weight), ("uk", self.wuk.t()),
            ("uv", self.wuv.weight), ("o", self.wo.weight)]

    def cache_spec(self):
        return LatentSpec(self.rank, self.rot)

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        rope = (cache.rope(self.rot_base, self.rot_dims, self.rot_scaling)
                if self.rot_dims else None)
        o = ops.latent_attention(
            ops.linear(h, self.win.weight), cache, run, plan,
            heads=self.heads, dim=self.dim, vdim=self.vdim, rot=self.rot,
            q_norm=self.q_norm, kv_norm=self.kv_norm, wuq=self.wuq.weight,
            wuk=self.wuk, wuv=self.wuv.weight, rope=rope, size=self.size,
            scale=self.scale, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class Mamba2(nn.Module):
    """State-space recurrence with a decay per head and token, a short
    causal convolution before it and a gated, grouped RMS norm after."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.vdim, self.n = (spec["heads"], spec["vdim"],
                                         spec["state"])
        self.groups, self.taps = spec["groups"], spec["conv"]
        self.parts = spec["norm_groups"]
        self.inner = self.heads * self.vdim
        self.channels = self.inner + 2 * self.groups * self.n
        if self.heads % self.groups:
            raise ValueError(f"groups {self.groups} must divide heads "
                             f"{self.heads}")
        if self.inner % self.parts:
            raise ValueError(f"norm_groups {self.parts} must divide "
                             f"{self.inner}")
        self.eps = eps
        # rows: gate z | x, B, C | step sizes
        self.rows = self.inner + self.channels + self.heads
        self.win = nn.Linear(width, _pad8(self.rows), bias=False)
        self.conv = nn.Parameter(torch.zeros(self.channels, self.taps))
        self.conv_b = nn.Parameter(torch.zeros(self.channels))
        self.dt_bias = nn.Parameter(torch.zeros(self.heads))
        self.a_log = nn.Parameter(torch.zeros(self.heads))
        self.skip = nn.Parameter(torch.ones(self.heads))
        self.norm = nn.Parameter(torch.ones(self.inner))
        self.wo = nn.Linear(self.inner, width, bias=False)

    def packed(self):
        return _cut(self.win.weight, **{"in": self.rows}) + [
            ("conv", self.conv), ("conv.b", self.conv_b),
            ("dt_bias", self.dt_bias), ("A_log", self.a_log),
            ("D", self.skip), ("norm", self.norm), ("o", self.wo.weight)]

    def cache_spec(self):
        return StateSpec(((self.heads, self.vdim, self.n),
                          (self.taps - 1, self.channels)))

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        o = ops.mamba2(
            ops.linear(h, self.win.weight), cache, run, plan,
            groups=self.groups, conv=self.conv, conv_b=self.conv_b,
            dt_bias=self.dt_bias, a_log=self.a_log, skip=self.skip,
            norm=self.norm, parts=self.parts, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class MLSTM(nn.Module):
    """Matrix memory with exponential input and sigmoid forget gates, kept
    in range by a running maximum; a per-head output norm and a sigmoid
    gate."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.dim, self.vdim = (spec["heads"], spec["dim"],
                                           spec["vdim"])
        self.cap = float(spec["gate_cap"])
        self.eps = eps
        # rows: q | k | v | output gate | input gate | forget gate
        self.win = nn.Linear(width, _pad8(
            2 * self.heads * (self.dim + self.vdim + 1)), bias=False)
        self.i_b = nn.Parameter(torch.zeros(self.heads))
        self.f_b = nn.Parameter(torch.zeros(self.heads))
        self.norm = nn.Parameter(torch.ones(self.heads * self.vdim))
        self.wo = nn.Linear(self.heads * self.vdim, width, bias=False)

    def packed(self):
        a, b = self.heads * self.dim, self.heads * self.vdim
        return _cut(self.win.weight, q=a, k=a, v=b, g=b, i=self.heads,
                    f=self.heads) + [
            ("i.b", self.i_b), ("f.b", self.f_b), ("norm", self.norm),
            ("o", self.wo.weight)]

    def cache_spec(self):
        # the memory (transposed), its normalizer and the running maximum
        return StateSpec(((self.heads, self.vdim, self.dim),
                          (self.heads, self.dim), (self.heads,)))

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        o = ops.mlstm(
            ops.linear(h, self.win.weight), cache, run, plan, i_b=self.i_b,
            f_b=self.f_b, cap=self.cap, norm=self.norm, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class Lightning(nn.Module):
    """Linear attention with a fixed decay per head, silu on queries, keys and
    values, one RMS norm over all heads and a sigmoid gate."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        self.heads, self.dim, self.vdim = (spec["heads"], spec["dim"],
                                           spec["vdim"])
        self.decay = [float(d) for d in spec["decay"]]
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} "
                             "heads")
        self.eps = eps
        # rows: q | k | v | gate
        self.win = nn.Linear(width, 2 * self.heads * (self.dim + self.vdim),
                             bias=False)
        self.norm = nn.Parameter(torch.ones(self.heads * self.vdim))
        self.wo = nn.Linear(self.heads * self.vdim, width, bias=False)
        self._tables = {}      # device -> decay tables (always float32)

    def packed(self):
        a, b = self.heads * self.dim, self.heads * self.vdim
        return (_cut(self.win.weight, q=a, k=a, v=b, g=b)
                + [("norm", self.norm), ("o", self.wo.weight)])

    def cache_spec(self):
        return StateSpec(((self.heads, self.vdim, self.dim),))

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        key = str(h.device)
        if key not in self._tables:
            self._tables[key] = ops.decay_tables(self.decay, TILE, h.device)
        pows, dec = self._tables[key]
        o = ops.lightning(ops.linear(h, self.win.weight), cache, run, plan,
                          pows=pows, dec=dec, norm=self.norm, eps=self.eps)
        return ops.linear(o, self.wo.weight)


class _Branch(nn.Module):
    """A mixer that can stand alone or share its input and output matrices
    with others (Parallel): it reads `rows` outputs of an input matrix and
    writes `cols` columns that an output matrix reads (mix)."""

    def _matrices(self, width: int, shared: bool) -> None:
        if not shared:
            self.win = nn.Linear(width, _pad8(self.rows), bias=False)
            self.wo = nn.Linear(self.cols, width, bias=False)

    def packed(self):
        return self.views(self.win.weight, self.wo.weight)

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        out = h.new_empty(h.shape[0], self.cols)
        self.mix(ops.linear(h, self.win.weight), 0, out, 0, 1.0, plan, cache,
                 run)
        return ops.linear(out, self.wo.weight)


class WindowAttention(_Branch):
    """Grouped-query attention over a sliding window of mask.size tokens and
    the first mask.keep_first ones, without rotation: soft-capped scores take
    a learned bias by distance (`buckets` rows, the last from bias_max on);
    values are divided by their root mean square; a sigmoid gate per
    element."""

    def __init__(self, width: int, spec: dict, eps: float,
                 shared: bool = False):
        super().__init__()
        self.heads, self.kv = spec["heads"], spec["kv_heads"]
        self.dim, self.vdim = spec["dim"], spec["vdim"]
        self.scale = float(spec["scale"])
        self.softcap = float(spec.get("softcap") or 0.0)
        mask = spec.get("mask") or {}
        self.size = int(mask.get("size") or 0)
        self.keep = int(mask.get("keep_first") or 0)
        self.far, self.eps = int(spec["bias_max"]), eps
        if self.heads % self.kv:
            raise ValueError(f"kv_heads {self.kv} must divide heads "
                             f"{self.heads}")
        if not 1 <= spec["buckets"] // 2 < self.far:
            raise ValueError(f"bias_max {self.far} must be above half of "
                             f"{spec['buckets']} buckets, at least two")
        # q | k | v | gate
        self.parts = {"q": self.heads * self.dim, "k": self.kv * self.dim,
                      "v": self.kv * self.vdim, "g": self.heads * self.vdim}
        self.rows, self.cols = sum(self.parts.values()), self.parts["g"]
        self._matrices(width, shared)
        self.rel = nn.Parameter(torch.zeros(spec["buckets"], self.heads))
        self._bias = (None, None)    # what it was made from, bias by distance

    def views(self, win, wo):
        return _cut(win, **self.parts) + [("rel", self.rel), ("o", wo)]

    def cache_spec(self):
        return KVSpec(self.kv, self.dim, self.vdim)

    def mix(self, p, col, out, out_col, scale, plan: StepPlan,
            cache: PagedStateCache, run: int):
        key = (self.rel.data_ptr(), self.rel._version, p.device)
        if self._bias[0] != key:
            self._bias = key, ops.distance_bias(self.rel, self.far)
        ops.window_attention(
            p, col, out, out_col, cache, run, plan, heads=self.heads,
            bias=self._bias[1], softcap=self.softcap, size=self.size,
            keep=self.keep, scale=self.scale, out_scale=scale, eps=self.eps)


class GatedLinearAttention(_Branch):
    """Linear attention with a decay per key channel and token, made by a
    low-rank projection (`rank`), a per-head RMS norm and a silu gate."""

    def __init__(self, width: int, spec: dict, eps: float,
                 shared: bool = False):
        super().__init__()
        self.heads, self.dim, self.vdim = (spec["heads"], spec["dim"],
                                           spec["vdim"])
        self.rank, self.tau = spec["rank"], float(spec["tau"])
        self.eps = eps
        a, b = self.heads * self.dim, self.heads * self.vdim
        # q | k | v | gate | the decay's first projection
        self.parts = {"q": a, "k": a, "v": b, "g": b, "a1": self.rank}
        self.rows, self.cols = sum(self.parts.values()), b
        self._matrices(width, shared)
        self.a2 = nn.Parameter(torch.zeros(a, self.rank))
        self.a2_b = nn.Parameter(torch.zeros(a))
        self.norm = nn.Parameter(torch.ones(self.vdim))

    def views(self, win, wo):
        return _cut(win, **self.parts) + [
            ("a2", self.a2), ("a2.b", self.a2_b), ("norm", self.norm),
            ("o", wo)]

    def cache_spec(self):
        # transposed, [vdim][dim]: the order the kernels read
        return StateSpec(((self.heads, self.vdim, self.dim),))

    def mix(self, p, col, out, out_col, scale, plan: StepPlan,
            cache: PagedStateCache, run: int):
        ops.gla(p, col, out, out_col, cache, run, plan, rank=self.rank,
                a2=self.a2, a2_b=self.a2_b, tau=self.tau, norm=self.norm,
                out_scale=scale, eps=self.eps)


class Parallel(nn.Module):
    """Two mixers side by side, `left` and `right` (each a spec with a type),
    that read the same input; their results are summed with left_scale and
    right_scale.  One matrix projects the input for both, one sums both
    outputs; the scales join the epilogues."""

    def __init__(self, width: int, spec: dict, eps: float):
        super().__init__()
        for side in ("left", "right"):
            s = spec[side]
            kind = BRANCHES.get(s["type"])
            if kind is None:
                raise ValueError(f"{s['type']!r} cannot share its input "
                                 f"(known: {', '.join(sorted(BRANCHES))})")
            setattr(self, side, kind(width, s, eps, shared=True))
        self.scales = float(spec["left_scale"]), float(spec["right_scale"])
        self.split = _pad8(self.left.rows)    # where the right one's rows start
        self.win = nn.Linear(width, self.split + _pad8(self.right.rows),
                             bias=False)
        self.wo = nn.Linear(self.left.cols + self.right.cols, width,
                            bias=False)

    def packed(self):
        w, o, n = self.win.weight, self.wo.weight, self.left.cols
        return ([("left." + k, t)
                 for k, t in self.left.views(w[:self.split], o[:, :n])]
                + [("right." + k, t)
                   for k, t in self.right.views(w[self.split:], o[:, n:])])

    def cache_spec(self):
        return self.left.cache_spec(), self.right.cache_spec()

    def step(self, h, plan: StepPlan, cache: PagedStateCache, run: int):
        p = ops.linear(h, self.win.weight)
        out = h.new_empty(h.shape[0], self.wo.in_features)
        self.left.mix(p, 0, out, 0, self.scales[0], plan, cache, run)
        self.right.mix(p, self.split, out, self.left.cols, self.scales[1],
                       plan, cache, run)
        return ops.linear(out, self.wo.weight)


class DenseFF(nn.Module):
    def __init__(self, width: int, spec: dict, vocab: int = 0):
        super().__init__()
        self.up = nn.Linear(width, spec["ff"], bias=False)
        self.down = nn.Linear(spec["ff"], width, bias=False)

    def packed(self):
        return [("up", self.up.weight), ("down", self.down.weight)]

    def step(self, h, plan: StepPlan):
        return ops.linear(ops.gelu_erf(ops.linear(h, self.up.weight)),
                          self.down.weight)


class GatedFF(nn.Module):
    """down(gelu(gate x) * up x), the tanh form of GELU."""

    def __init__(self, width: int, spec: dict, vocab: int = 0):
        super().__init__()
        self.gate_up = nn.Linear(width, 2 * spec["ff"], bias=False)
        self.down = nn.Linear(spec["ff"], width, bias=False)

    def packed(self):
        ff = self.down.weight.shape[1]
        return (_cut(self.gate_up.weight, gate=ff, up=ff)
                + [("down", self.down.weight)])

    def step(self, h, plan: StepPlan):
        return ops.linear(ops.geglu_tanh(ops.linear(h, self.gate_up.weight)),
                          self.down.weight)


class ClampedFF(GatedFF):
    """down(g sigmoid(alpha g) (u + shift)), g = gate x cut off above
    `limit`, u = up x on both sides."""

    def __init__(self, width: int, spec: dict, vocab: int = 0):
        super().__init__(width, spec)
        self.limit, self.alpha, self.shift = (
            float(spec["limit"]), float(spec.get("alpha", 1.702)),
            float(spec.get("shift", 1.0)))

    def step(self, h, plan: StepPlan):
        a = ops.clamped_glu(ops.linear(h, self.gate_up.weight), self.limit,
                            self.alpha, self.shift)
        return ops.linear(a, self.down.weight)


class _Experts(nn.Module):
    """Many gated experts, each down(silu(gate x) * up x)."""

    def __init__(self, width: int, spec: dict):
        super().__init__()
        self.experts, self.top = spec["router"]["experts"], spec["router"]["top"]
        ff = spec["expert"]["ff"]
        self.gate_up = nn.Parameter(torch.empty(self.experts, 2 * ff, width))
        self.down = nn.Parameter(torch.empty(self.experts, width, ff))

    def packed(self):
        ff, out = self.down.shape[2], []
        for e in range(self.experts):
            out += _cut(self.gate_up[e], **{f"e{e}.gate": ff, f"e{e}.up": ff})
            out.append((f"e{e}.down", self.down[e]))
        return out


class RoutedFF(_Experts):
    """`top` of many gated experts per token, chosen by sigmoid scores out
    of the best groups of experts, and (spec["shared"]) an expert for every
    token, behind a gate.  Returns Parts: the residual norm sums them."""

    def __init__(self, width: int, spec: dict, vocab: int = 0):
        super().__init__(width, spec)
        r, sh = spec["router"], spec.get("shared")
        groups = r.get("groups") or {"count": 1, "keep": 1}
        self.groups, self.keep = groups["count"], groups["keep"]
        self.scale = float(r.get("scale", 1.0))
        E = self.experts
        if E % self.groups:
            raise ValueError(f"groups.count {self.groups} must divide "
                             f"experts {E}")
        if not 1 <= self.keep <= self.groups:
            raise ValueError(f"groups.keep {self.keep} of {self.groups}")
        if not 1 <= self.top <= self.keep * (E // self.groups):
            raise ValueError(f"top {self.top}: {self.keep} groups of "
                             f"{E // self.groups} experts to choose from")
        # rows: a logit per expert | the shared expert's gate
        self.router = nn.Linear(width, _pad8(E + (sh is not None)), bias=False)
        self.shared = None if sh is None else GatedFF(width, sh)

    def packed(self):
        E, out = self.experts, super().packed()
        out.append(("router", self.router.weight[:E]))
        if self.shared is not None:
            out += [(f"shared.{n}", t) for n, t in self.shared.packed()]
            out.append(("shared.sg", self.router.weight[E:E + 1]))
        return out

    def step(self, h, plan: StepPlan):
        sh = self.shared
        return ops.moe(h, self.router.weight, self.gate_up, self.down,
                       sh and (sh.gate_up.weight, sh.down.weight),
                       top=self.top, groups=self.groups, keep=self.keep,
                       scale=self.scale)


class TableFF(_Experts):
    """`top` of many gated experts per token, named by a table of token ids,
    with equal weights.  Returns Parts: the residual norm sums them."""

    def __init__(self, width: int, spec: dict, vocab: int = 0):
        super().__init__(width, spec)
        if not 1 <= self.top <= self.experts:
            raise ValueError(f"top {self.top} of {self.experts} experts")
        self.register_buffer("table", torch.rand(vocab, self.experts)
                             .argsort(1)[:, :self.top].to(torch.int32)
                             .contiguous())

    def packed(self):
        return super().packed() + [("table", self.table)]

    def check(self):
        """Refuse a loaded table that names an expert that is not there, or
        one twice for a token."""
        t = self.table.sort(1).values
        if t.numel() and (t.min() < 0 or t.max() >= self.experts
                          or (t[:, 1:] == t[:, :-1]).any()):
            raise ValueError(f"table: {self.top} different experts of "
                             f"{self.experts} expected per token")

    def step(self, h, plan: StepPlan):
        return ops.table_moe(h, plan.tokens, self.table, self.gate_up,
                             self.down)


MIXERS = {"attention": ChunkAttention, "tied_attention": TiedAttention,
          "retention": Retention, "latent_attention": LatentAttention,
          "mamba2": Mamba2, "mlstm": MLSTM, "lightning": Lightning,
          "window_attention": WindowAttention, "gla": GatedLinearAttention,
          "parallel": Parallel}
BRANCHES = {k: m for k, m in MIXERS.items() if issubclass(m, _Branch)}
FEED_FORWARDS = {"dense": DenseFF, "gated": GatedFF, "clamped": ClampedFF,
                 "moe": RoutedFF, "table_moe": TableFF}
