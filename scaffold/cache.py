"""Paged key/value pool and recurrent-state slots for mixer-stack models,
and the step plan that tells the kernels where a ragged batch's tokens
live.

A sequence owns one SLOT and a list of 64-token PAGES.  The page list is
shared by all attention layer runs (each has its own key/value or latent
tensors of the same page count); a recurrent layer run keeps one state per
slot, which may consist of several tensors.
Layers that run several times in a forward pass are separate runs here,
so every pass has its own keys, values and state.  A layer may have both
pages and a state; what a model keeps of a sequence beside its mixers (the
previous token, the inputs that a shift looks back at) are runs of their own.

A freed page or slot is handed out again as it is: nothing is cleared.
Kernels never read a key that the sequence did not write, and a sequence
that starts (position 0) starts its states from zero.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np
import torch

PAGE = 64   # tokens per page
TILE = 64   # prompt tokens per kernel tile
BLOCK = 128  # prompt tokens per block of attention over expanded keys


@dataclass(frozen=True)
class KVSpec:
    """What one run of an attention layer caches per token."""
    kv_heads: int
    dim: int
    vdim: int


@dataclass(frozen=True)
class TiedSpec:
    """What one run of an attention layer caches per token whose values are
    its keys: one row per head, and a float32 factor that norms them."""
    kv_heads: int
    dim: int


@dataclass(frozen=True)
class LatentSpec:
    """What one run of a latent-attention layer caches per token: a latent
    that keys and values are made from, and a rotated key part that all
    heads share.  Both are padded to multiples of 8 elements."""
    rank: int
    rot: int

    @property
    def row(self) -> int:
        return _pad8(self.rank) + _pad8(self.rot)


@dataclass(frozen=True)
class StateSpec:
    """What one run of a recurrent layer keeps per sequence: tensors of
    these shapes, float32 unless said otherwise."""
    shapes: Tuple[Tuple[int, ...], ...]
    dtype: torch.dtype = torch.float32


def _pad8(n: int) -> int:
    return -(-n // 8) * 8


class CacheFull(RuntimeError):
    """No free slot or not enough free pages."""


@dataclass
class StepPlan:
    """One ragged batch.  Rows [0, n_dec) are single tokens, each of its
    own sequence; the rest are prompt portions, tile by tile.

    tiles (n, 4): first row, rows (<= TILE), position of the first, slot
    seqs  (m, 4): first tile, tiles, position of the portion, slot
    slot < 0 marks a row to skip (an idle slot of a fixed-width step).
    portions repeats the prompt portions for the host: first row, rows,
    position of the first, slot."""
    tokens: torch.Tensor           # (T,) int64
    pos: torch.Tensor              # (T,) int32
    slot: torch.Tensor             # (T,) int32
    tiles: torch.Tensor
    seqs: torch.Tensor
    n_dec: int
    rows: Optional[torch.Tensor]   # wanted rows, int32; None = every row
    portions: Sequence[Tuple[int, int, int, int]] = ()
    _spans: Dict[int, Tuple[torch.Tensor, torch.Tensor]] = field(
        default_factory=dict)

    def spans(self, size: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """The keys that the portions see through a sliding window of
        `size` tokens (0: every earlier one), laid out one portion after
        the other, and the portions' rows cut into blocks:

        keys   (R, 4): batch row (-1: a cached token), slot, position, 0
        blocks (n, 4): first row, rows (<= BLOCK), position of the first,
                       place of position 0 among the keys"""
        if size not in self._spans:
            keys, blocks, at = [], [], 0
            for row, n, p0, slot in self.portions:
                lo = max(0, p0 - size + 1) if size else 0
                p = np.arange(lo, p0 + n)
                k = np.zeros((p.size, 4), np.int32)
                k[:, 0] = np.where(p < p0, -1, row + p - p0)
                k[:, 1] = slot
                k[:, 2] = p
                keys.append(k)
                blocks.extend((row + o, min(BLOCK, n - o), p0 + o, at - lo)
                              for o in range(0, n, BLOCK))
                at += p.size
            flat = np.concatenate([np.asarray(blocks, np.int32).reshape(-1)]
                                  + [k.reshape(-1) for k in keys])
            dev = torch.from_numpy(flat).to(self.pos.device)
            b, k = torch.split(dev, [4 * len(blocks), 4 * at])
            self._spans[size] = k.view(at, 4), b.view(len(blocks), 4)
        return self._spans[size]


# (slot, tokens, want): tokens is a list of ids or a 1-D device tensor,
# want the places among them whose logits are asked for
Entry = Tuple[int, object, Sequence[int]]


class PagedStateCache:
    def __init__(self, specs: Sequence[object], n_slots: int, n_tokens: int,
                 max_len: int, device, dtype):
        """specs: one per run, or a tuple of them (one of what tokens leave
        in pages, any of what a sequence keeps); n_tokens: pool size in tokens
        (rounded up to whole pages); max_len: the longest sequence a slot can
        hold."""
        self.device = torch.device(device)
        self.specs = list(specs)
        self.n_slots = n_slots
        self.n_pages = -(-n_tokens // PAGE)
        self.max_len = max_len
        self.max_pages = max(1, -(-max_len // PAGE))
        self.k: List[Optional[torch.Tensor]] = []
        self.v: List[Optional[torch.Tensor]] = []
        self.state: List[Optional[Tuple[torch.Tensor, ...]]] = []
        for spec in self.specs:
            k = v = state = None
            for s in spec if isinstance(spec, tuple) else (spec,):
                if isinstance(s, StateSpec):
                    state = (state or ()) + tuple(
                        torch.zeros(n_slots, *shape, device=device,
                                    dtype=s.dtype) for shape in s.shapes)
                    continue
                if k is not None:
                    raise ValueError("a run has one cache of tokens")
                if isinstance(s, LatentSpec):
                    k = torch.zeros(self.n_pages, PAGE, s.row, device=device,
                                    dtype=dtype)
                    continue
                k = torch.zeros(self.n_pages, s.kv_heads, PAGE, s.dim,
                                device=device, dtype=dtype)
                if isinstance(s, KVSpec):
                    v = torch.zeros(self.n_pages, s.kv_heads, PAGE, s.vdim,
                                    device=device, dtype=dtype)
                else:
                    v = torch.zeros(self.n_pages, PAGE, device=device,
                                    dtype=torch.float32)
            self.k.append(k)
            self.v.append(v)
            self.state.append(state)
        self.table = torch.zeros(n_slots, self.max_pages, dtype=torch.int32,
                                 device=device)
        self._pages: List[List[int]] = [[] for _ in range(n_slots)]
        self._free_pages = list(range(self.n_pages - 1, -1, -1))
        self._open = [False] * n_slots
        self.lens = [0] * n_slots
        self._rope: Dict[tuple, Tuple[torch.Tensor, torch.Tensor]] = {}
        self._none4 = torch.zeros(0, 4, dtype=torch.int32, device=device)

    # ---- slots and pages ------------------------------------------------
    def open(self, slot: Optional[int] = None) -> int:
        if slot is None:
            slot = next((i for i, o in enumerate(self._open) if not o), -1)
            if slot < 0:
                raise CacheFull(f"all {self.n_slots} slots are in use")
        elif self._open[slot]:
            raise ValueError(f"slot {slot} is in use")
        self._open[slot] = True
        self.lens[slot] = 0
        return slot

    def close(self, slot: int) -> None:
        if not self._open[slot]:
            raise ValueError(f"slot {slot} is not open")
        self._open[slot] = False
        self._free_pages.extend(reversed(self._pages[slot]))
        self._pages[slot] = []
        self.lens[slot] = 0

    @property
    def free_tokens(self) -> int:
        return len(self._free_pages) * PAGE

    def pages_for(self, n: int) -> int:
        return -(-n // PAGE)

    def reserve(self, slot: int, n: int) -> None:
        """Give the slot pages for its first n tokens."""
        if not self._open[slot]:
            raise ValueError(f"slot {slot} is not open")
        if n > self.max_len:
            raise ValueError(f"{n} tokens exceed max_len {self.max_len}")
        own = self._pages[slot]
        add = self.pages_for(n) - len(own)
        if add <= 0:
            return
        if add > len(self._free_pages):
            raise CacheFull(f"{add} pages wanted, {len(self._free_pages)} free")
        lo = len(own)
        own.extend(self._free_pages.pop() for _ in range(add))
        self.table[slot, lo:len(own)] = torch.tensor(
            own[lo:], dtype=torch.int32).to(self.device)

    # ---- one rectangular batch (row b is slot b) ------------------------
    @property
    def seq_len(self) -> int:
        return self.lens[0]

    @property
    def len(self) -> int:
        return self.lens[0]

    # ---- snapshots: reuse of a prompt, and stepping back ----------------
    def snapshot(self, slot: int, kv: bool = True) -> dict:
        """The slot's states and (kv) its keys and values, copied."""
        n = self.lens[slot]
        pages = torch.tensor(self._pages[slot][:self.pages_for(n)],
                             dtype=torch.int64, device=self.device)
        snap = {"len": n, "state": [None if s is None else
                                    tuple(t[slot].clone() for t in s)
                                    for s in self.state]}
        if kv:
            snap["k"] = [None if t is None else t[pages] for t in self.k]
            snap["v"] = [None if t is None else t[pages] for t in self.v]
        return snap

    def restore(self, slot: int, snap: dict) -> None:
        n = snap["len"]
        for mine, kept in zip(self.state, snap["state"]):
            for s, t in zip(mine or (), kept or ()):
                s[slot].copy_(t)
        if "k" in snap:
            self.reserve(slot, n)
            pages = torch.tensor(self._pages[slot][:self.pages_for(n)],
                                 dtype=torch.int64, device=self.device)
            for dst, src in ((self.k, snap["k"]), (self.v, snap["v"])):
                for d, s in zip(dst, src):
                    if d is not None:
                        d[pages] = s
        self.lens[slot] = n

    # ---- rotary tables --------------------------------------------------
    def rope(self, base: float, dims: int, scaling: Optional[dict] = None):
        """cos/sin (max_len, dims/2) float32 of position * base^(-2i/dims),
        angles taken in float64; scaling: YaRN's constants."""
        key = (base, dims, tuple(sorted((scaling or {}).items())))
        if key not in self._rope:
            from . import ops

            self._rope[key] = ops.rope_tables_exact(self.max_len, dims, base,
                                                    self.device, scaling)
        return self._rope[key]

    # ---- step plans -----------------------------------------------------
    def plan(self, entries: Sequence[Entry]) -> Tuple[StepPlan, List[int]]:
        """Reserve pages for a ragged batch and lay it out.  Returns the
        plan and the number of wanted rows per entry (the plan's rows
        follow the entries' order).  Call commit() after the step ran."""
        sizes = []
        need = 0
        for slot, toks, want in entries:
            n = toks.numel() if torch.is_tensor(toks) else len(toks)
            if n == 0:
                raise ValueError("an entry needs at least one token")
            if any(not 0 <= w < n for w in want):
                raise ValueError("wanted place outside the entry's tokens")
            if self.lens[slot] + n > self.max_len:
                raise ValueError(f"{self.lens[slot] + n} tokens exceed "
                                 f"max_len {self.max_len}")
            need += max(0, self.pages_for(self.lens[slot] + n)
                        - len(self._pages[slot]))
            sizes.append(n)
        if len({e[0] for e in entries}) != len(entries):
            raise ValueError("a sequence may have one entry per step")
        if need > len(self._free_pages):
            raise CacheFull(f"{need} pages wanted, "
                            f"{len(self._free_pages)} free")
        T = sum(sizes)
        tok = np.zeros(T, np.int32)
        pos = np.zeros(T, np.int32)
        slots = np.zeros(T, np.int32)
        tiles, seqs, portions = [], [], []
        first = [0] * len(entries)
        from_device = []
        at = n_dec = 0
        # single tokens first, portions after them
        for i in sorted(range(len(entries)), key=lambda i: sizes[i] > 1):
            slot, toks, _ = entries[i]
            n, p0 = sizes[i], self.lens[slot]
            self.reserve(slot, p0 + n)
            first[i] = at
            if torch.is_tensor(toks):
                from_device.append((at, n, toks))
            else:
                tok[at:at + n] = toks
            pos[at:at + n] = np.arange(p0, p0 + n)
            slots[at:at + n] = slot
            if n == 1:
                n_dec += 1
            else:
                portions.append((at, n, p0, slot))
                seqs.append((len(tiles), -(-n // TILE), p0, slot))
                tiles.extend((at + o, min(TILE, n - o), p0 + o, slot)
                             for o in range(0, n, TILE))
            at += n
        rows = [first[i] + w for i, e in enumerate(entries) for w in e[2]]
        # one upload; the int4 lists come first so they stay 16-byte aligned
        nt, ns = len(tiles), len(seqs)
        flat = np.concatenate([
            np.asarray(tiles, np.int32).reshape(-1),
            np.asarray(seqs, np.int32).reshape(-1), pos, slots, tok,
            np.asarray(rows, np.int32)])
        dev = torch.from_numpy(flat).to(self.device)
        cut = [4 * nt, 4 * ns, T, T, T, len(rows)]
        tl, sq, ps, sl, tk, rw = torch.split(dev, cut)
        tokens = tk.long()
        for a, n, src in from_device:
            tokens[a:a + n] = src.view(-1)
        return (StepPlan(tokens, ps, sl, tl.view(nt, 4), sq.view(ns, 4),
                         n_dec, rw, portions), [len(e[2]) for e in entries])

    def commit(self, entries: Sequence[Entry]) -> None:
        for slot, toks, _ in entries:
            self.lens[slot] += (toks.numel() if torch.is_tensor(toks)
                                else len(toks))

    def decode_plan(self, tokens: torch.Tensor, pos: torch.Tensor,
                    active: Optional[torch.Tensor] = None) -> StepPlan:
        """Fixed-width plan: row b is slot b's next token at pos[b]; rows
        with active[b] == 0 are skipped.  Device work only, so a step
        built on it can be captured in a graph; the caller has reserved
        the pages and advances `lens` (advance())."""
        B = tokens.numel()
        slot = torch.arange(B, dtype=torch.int32, device=self.device)
        if active is not None:
            slot = torch.where(active.view(-1) > 0, slot,
                               torch.full_like(slot, -1))
        return StepPlan(tokens.reshape(-1), pos.reshape(-1).to(torch.int32),
                        slot, self._none4, self._none4, B, None)

    def advance(self, slots: Sequence[int], n: int = 1) -> None:
        for s in slots:
            self.lens[s] += n
