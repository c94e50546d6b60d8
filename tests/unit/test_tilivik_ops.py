"""Each mechanism of the Tilivik design against the plain oracle: the
float32 forms on the CPU, the HIP kernels (float32 and bfloat16) on the
GPU.  Caches start full of NaN, and a sequence is fed in several cuts."""

import math

import pytest
import torch

from scaffold import ops
from tests.oracle import tilivik as O
from tests.oracle.cases import KVSpec, StateSpec, cuts, op_cache
from tests.oracle.places import close, gpu, place, rnd

PARTS = {"whole": lambda T: [T], "tokens": lambda T: [1] * T,
         "portions": lambda T: cuts(T, [2, 3, 61, 1, 64, 17])}
cut = pytest.mark.parametrize("parts", sorted(PARTS))


def scalar():
    """A norm's only weight."""
    return (rnd(1, seed=3)[0] + 2).bfloat16().double()


def feed(T, parts, cache, slot, tokens, run):
    """run(plan, first row, last row) over portions; its results in order."""
    outs, at = [], 0
    for n in parts:
        ent = [(slot, tokens[at:at + n], ())]
        plan, _ = cache.plan(ent)
        outs.append(run(plan, at, at + n))
        cache.commit(ent)
        at += n
    assert at == T
    return [torch.cat(o) for o in zip(*outs)]


# ------------------------------------------------------------------ embedding
def embed_case(W, V=23, buckets=31, seed=0):
    return {"cfg": {"width": W, "embedding": {"bigram": {
        "buckets": buckets, "mul_prev": 13, "mul_cur": 5}}},
        "w": {"embed": rnd(V, W, seed=seed),
              "bigram": rnd(buckets + 1, W, seed=seed + 1)}}


def run_embed(case, dev, dt, tokens, parts, cache=None, slot=None):
    w, spec = case["w"], case["cfg"]["embedding"]["bigram"]
    cache = cache or op_cache(StateSpec(((),), torch.int64), dev, dt)
    slot = cache.open() if slot is None else slot
    W = case["cfg"]["width"]
    got, = feed(len(tokens), parts, cache, slot, tokens, lambda plan, a, b: [
        ops.stream_embed(plan, w["embed"].to(dev, dt),
                         rates=ops.turn_rates(W, 10000.0, dev),
                         pairs=w["bigram"].to(dev, dt),
                         mul=(spec["mul_prev"], spec["mul_cur"]),
                         last=cache.state[0][0])])
    return got


@place
@cut
@pytest.mark.parametrize("W", [8, 37, 260, 1030])
def test_embeddings_of_pairs_and_positions(dev, dt, W, parts):
    case, T = embed_case(W), 150
    g = torch.Generator().manual_seed(W)
    tokens = torch.randint(0, 23, (T,), generator=g).tolist()
    got = run_embed(case, dev, dt, tokens, PARTS[parts](T))
    assert got.dtype == torch.float32
    close(got, O.embedding(case["cfg"], case["w"], tokens), torch.float32)


@place
def test_a_token_before_belongs_to_its_sequence(dev, dt):
    """Neighbours in a batch, and whoever had the slot before, do not."""
    case = embed_case(20)
    seqs = [[3, 7, 7, 1, 0], [7, 7], [22]]
    cache = op_cache(StateSpec(((),), torch.int64), dev, dt)
    for s in seqs:                                    # slots used before
        run_embed(case, dev, dt, [9, 4, 8], [2, 1], cache, cache.open())
    for s in range(3):
        cache.close(s)
    slots = [cache.open() for _ in seqs]
    entries = [(slots[i], s, ()) for i, s in enumerate(seqs)]
    plan, _ = cache.plan(entries)
    w, spec = case["w"], case["cfg"]["embedding"]["bigram"]
    got = ops.stream_embed(
        plan, w["embed"].to(dev, dt), rates=ops.turn_rates(20, 10000.0, dev),
        pairs=w["bigram"].to(dev, dt),
        mul=(spec["mul_prev"], spec["mul_cur"]), last=cache.state[0][0])
    # single tokens come first in a plan
    want = torch.cat([O.embedding(case["cfg"], w, seqs[i]) for i in (2, 0, 1)])
    close(got, want, torch.float32)


@place
def test_far_positions_keep_their_digits(dev, dt):
    """One token at a position where float angles have lost theirs."""
    W, p = 64, 900_001
    cache = op_cache(StateSpec(((),), torch.int64), dev, dt, slots=1)
    plan = cache.decode_plan(torch.tensor([[2]], device=dev),
                             torch.tensor([p], device=dev))
    x = ops.stream_embed(plan, torch.zeros(5, W, device=dev, dtype=dt),
                         rates=ops.turn_rates(W, 10000.0, dev))
    close(x[0], O.sinusoid(p, W), torch.float32, 0.05)


# ------------------------------------------------------- norms that look back
def run_shift(dev, dt, x, parts, norm, eps, shift, *, y=None, add=None,
              step=None, mult=1.0, cache=None, slot=None):
    T, W = x.shape
    to = lambda t: t.to(dev, dt)
    cache = cache or op_cache(StateSpec(((W,),)), dev, dt)
    slot = cache.open() if slot is None else slot

    def run(plan, a, b):
        part = None if y is None else (
            ops.Parts(to(y[0][a:b]).contiguous(), y[1][a:b].float().to(dev))
            if isinstance(y, tuple) else to(y[a:b]))
        return ops.shift_norm(
            x[a:b].float().to(dev), part, mult, tuple(map(to, norm)), eps,
            plan, shift=to(shift), state=cache.state[0][0],
            add=None if add is None else add[a:b].float().to(dev),
            step=None if step is None else to(step))

    return feed(T, parts, cache, slot, [0] * T, run)


@place
@cut
@pytest.mark.parametrize("W", [8, 37, 256, 300, 1030, 2048, 4100])
def test_token_shift_of_a_scalar_norm(dev, dt, W, parts):
    """One weight for all columns; the blend is of normed vectors."""
    T, eps = 70 if parts == "tokens" else 141, 0.03
    x, y, g = rnd(T, W, seed=1, scale=3), rnd(T, 2, W, seed=2), scalar()
    c, add, step = rnd(T, 2, seed=4), rnd(T, W, seed=5), rnd(W, seed=6)
    mix = rnd(W, seed=7)
    z, h = run_shift(dev, dt, x, PARTS[parts](T), (g,), eps, mix, y=(y, c),
                     add=add, step=step, mult=0.7)
    want = x + 0.7 * (y * c.unsqueeze(2)).sum(1) + add + step
    assert z.dtype == torch.float32 and h.dtype == dt
    close(z, want, torch.float32)
    close(h, O.token_shift(O.rms(want, eps) * g, mix), dt)


@place
@pytest.mark.parametrize("n", [600, 2600, 5000])
def test_token_shift_of_long_portions(dev, dt, n):
    """More rows than a group walks alone, two sequences side by side."""
    if dev == "cpu":
        n //= 10
    W, eps = 12, 1e-3
    cache = op_cache(StateSpec(((W,),)), dev, dt, n_tokens=16384, max_len=8192)
    lens = [n, 3, n // 2 + 1, 1][:3]
    x, g, mix = rnd(sum(lens), W, seed=1), scalar(), rnd(W, seed=7)
    plan, _ = cache.plan([(cache.open(), [0] * k, ()) for k in lens])
    _, h = ops.shift_norm(x.float().to(dev), None, 1.0, (g.to(dev, dt),), eps,
                          plan, shift=mix.to(dev, dt), state=cache.state[0][0])
    at = 0
    for s, k in enumerate(lens):
        u = O.rms(x[at:at + k], eps) * g
        close(h[at:at + k], O.token_shift(u, mix), dt)
        close(cache.state[0][0][s], u[-1], torch.float32)
        at += k


@place
def test_shift_state_is_the_unblended_vector(dev, dt):
    """What is kept is the norm itself, of the last token, for each slot; a
    sequence starts from zeros whoever had the slot."""
    W, eps = 16, 1e-5
    x, g, mix = rnd(5, W, seed=1), scalar(), rnd(W, seed=7)
    cache = op_cache(StateSpec(((W,),)), dev, dt)
    s = cache.open()
    _, h = run_shift(dev, dt, x, [2, 1, 2], (g,), eps, mix, cache=cache, slot=s)
    u = O.rms(x, eps) * g
    close(cache.state[0][0][s], u[-1], torch.float32)
    cache.close(s)
    _, h = run_shift(dev, dt, x, [1, 4], (g,), eps, mix, cache=cache,
                     slot=cache.open())
    close(h, O.token_shift(u, mix), dt)


@place
def test_scalar_norm_between_sublayers(dev, dt):
    for W in (10, 256, 2052):
        x, y, g = rnd(4, W, seed=1), rnd(4, W, seed=2), scalar()
        xs = x.float().to(dev)
        h = ops.residual_norm(xs, y.to(dev, dt), None, 1.0, (g.to(dev, dt),),
                              0.01)
        close(xs, x + y, torch.float32)
        close(h, O.rms(x + y, 0.01) * g, dt)


# ---------------------------------------------------------------- attention
def run_window(dev, dt, q, k, v, gate, rel, mx, parts, eps=1e-6, scale=1.0,
               cache=None, slot=None):
    """Through the op in portions, among other columns of x and out."""
    T, H, d = q.shape
    G, e = v.shape[1:]
    cache = cache or op_cache(KVSpec(G, d, e), dev, dt)
    slot = cache.open() if slot is None else slot
    x = torch.cat([t.reshape(T, -1) for t in (q, k, v, gate)], 1)
    x = torch.nn.functional.pad(x, (8, -x.shape[1] % 8), value=float("nan"))
    x = x.to(dev, dt)
    mask = mx.get("mask") or {}
    bias = ops.distance_bias(rel.to(dev, dt), mx["bias_max"])

    def run(plan, a, b):
        out = torch.full((b - a, H * e + 5), 7.0, device=dev, dtype=dt)
        ops.window_attention(
            x[a:b].contiguous(), 8, out, 4, cache, 0, plan, heads=H,
            bias=bias, softcap=mx["softcap"], size=mask.get("size", 0),
            keep=mask.get("keep_first", 0), scale=mx["scale"],
            out_scale=scale, eps=eps)
        assert (out[:, :4] == 7).all() and (out[:, -1] == 7).all()
        return [out[:, 4:-1]]

    got, = feed(T, parts, cache, slot, [0] * T, run)
    return got.view(T, H, e)


def want_window(q, k, v, gate, rel, mx, eps=1e-6, scale=1.0, rows=0):
    o = O.window_attention(q[rows:], k, O.rms(v, eps), rel, mx, rows)
    return o * O.sigmoid(gate[rows:].reshape(o.shape)) * scale


def window_case(H, G, d, e, T, rows=14, far=40, size=50, keep=3, cap=5.0,
                seed=0):
    q, k = rnd(T, H, d, seed=seed + 1), rnd(T, G, d, seed=seed + 2)
    v = rnd(T, G, e, seed=seed + 3)
    v = (v * torch.linspace(0.2, 3, T, dtype=torch.float64).view(-1, 1, 1)
         ).bfloat16().double()
    mx = {"scale": 1.5 * d ** -0.5, "softcap": cap, "bias_max": far,
          "mask": {"size": size, "keep_first": keep}}
    return q, k, v, rnd(T, H * e, seed=seed + 4), rnd(rows, H, seed=seed + 5), mx


SHAPES = [(4, 2, 16, 16), (3, 3, 9, 5), (8, 2, 128, 64), (2, 1, 256, 200),
          (12, 2, 64, 128), (5, 1, 40, 72), (4, 4, 32, 24), (7, 1, 64, 64),
          (1, 1, 1, 1)]


@place
@cut
@pytest.mark.parametrize("shape", SHAPES, ids=str)
def test_window_attention(dev, dt, shape, parts):
    case = window_case(*shape, T=131 if parts != "tokens" else 70)
    got = run_window(dev, dt, *case, PARTS[parts](case[0].shape[0]),
                     eps=0.01, scale=0.6)
    close(got, want_window(*case, eps=0.01, scale=0.6), dt)


@place
@pytest.mark.parametrize("size,keep", [(1, 0), (1, 1), (2, 5), (64, 0),
                                       (63, 64), (65, 65), (64, 130), (40, 7),
                                       (300, 2), (0, 0)])
def test_masks(dev, dt, size, keep):
    case = window_case(4, 2, 16, 16, T=200, size=size, keep=keep)
    want = want_window(*case)
    for parts in ([200], [130, 1, 69], cuts(200, [2]), [150] + [1] * 50):
        close(run_window(dev, dt, *case, parts), want, dt)


def one_key(where, T, size, keep, dim=32, far=40, cap=30.0):
    """The last query has one answer, at `where`; values tell which key
    was taken."""
    q, k, v, gate, rel, mx = window_case(8, 2, dim, 16, T, far=far, size=size,
                                         keep=keep, cap=cap)
    q, k, rel = q * 0.05, k * 0.3, rel * 0.1
    k[where] = 0
    k[where, :, 3] = 8.0
    q[-1, :, 3] = 8.0
    v[where] = 0
    v[where, :, 5] = 3.0
    mx["scale"] = 0.5
    gate = gate * 0 + 9.0
    return q, k, v, gate, rel, mx


@place
@pytest.mark.parametrize("where", [0, 1, 2, 3, 4, 62, 63, 64, 65, 127, 128, 192,
                                   198, 199, 200, 201, 298])
def test_one_key_at_every_edge(dev, dt, where):
    """Window 100 and 4 kept tokens: a key is found up to 99 back and among
    the first 4, and not one step beyond, in prompts, portions and by single
    tokens."""
    T = 300
    case = one_key(where, T, 100, 4)
    want = want_window(*case, rows=T - 1)
    found = where < 4 or T - 1 - where < 100
    assert (want[0, :, 5] > 3.0).all() == found
    for parts in ([T], [T - 1, 1], [T - 2, 2], cuts(T, [64]), [201, 98, 1]):
        close(run_window(dev, dt, *case, parts)[-1:], want, dt)


@place
@pytest.mark.parametrize("keep", [60, 64, 70, 190])
def test_kept_tokens_beside_and_under_the_window(dev, dt, keep):
    """Kept pages that touch or overlap the window's are read once."""
    case = window_case(4, 1, 64, 64, T=260, size=70, keep=keep)
    want = want_window(*case)
    for parts in ([260], [129, 130, 1], [200] + [1] * 60):
        close(run_window(dev, dt, *case, parts), want, dt)


@place
@pytest.mark.parametrize("rows,far", [(2, 3), (7, 9), (14, 40), (32, 128),
                                      (33, 700), (6, 2000)])
def test_distance_bias(dev, dt, rows, far):
    """Equal scores, so that the bias alone weighs: each row of the table
    has its distances, also far beyond the table's last."""
    T = 260
    q, k, v, gate, rel, mx = window_case(3, 1, 16, 24, T, rows=rows, far=far,
                                         size=0, keep=0)
    q, rel = q * 0, rel * 2
    table = ops.distance_bias(rel, far)
    assert table.shape == (3, far + 1)
    for n in (0, 1, rows // 2 - 1, rows // 2, far // 2, far - 1, far):
        assert torch.equal(table[:, n].double(), rel[O.bucket(n, rows, far)])
    case = q, k, v, gate, rel, mx
    want = want_window(*case)
    for parts in ([T], [200] + [1] * 60, cuts(T, [33])):
        close(run_window(dev, dt, *case, parts), want, dt)


@place
def test_bias_joins_after_the_cap_and_without_the_scale(dev, dt):
    case = window_case(4, 2, 16, 16, T=90, cap=0.7)
    q, k, v, gate, rel, mx = case
    q, rel = q * 4, rel * 3
    case = q, k, v, gate, rel, mx
    want = want_window(*case)
    wrong = want_window(q, k, v, gate, rel * mx["scale"], mx)
    assert (wrong - want).abs().max() > 0.1
    for parts in ([90], [1] * 90):
        close(run_window(dev, dt, *case, parts), want, dt)


@place
def test_loud_values_are_normed_in_the_cache(dev, dt):
    q, k, v, gate, rel, mx = window_case(2, 1, 16, 16, T=80)
    v[40] *= 1000
    v[41] *= 2.0 ** -12
    case = q, k, v.bfloat16().double(), gate, rel, mx
    cache = op_cache(KVSpec(1, 16, 16), dev, dt)
    got = run_window(dev, dt, *case, [40, 1, 39], eps=1e-9, cache=cache)
    close(got, want_window(*case, eps=1e-9), dt)
    page = cache._pages[0][0]
    close(cache.v[0][page, 0, 40:42], O.rms(case[2][40:42, 0], 1e-9), dt)
    close(cache.k[0][page, 0, :64], k[:64, 0], dt)


@gpu
@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
def test_long_decode_in_splits(dt):
    """Many keys, split over blocks, beside an idle row."""
    T, H, G, d = 2100, 8, 2, 64
    case = window_case(H, G, d, d, T, rows=32, far=128, size=1500, keep=5)
    want = want_window(*case, rows=T - 3)
    got = run_window("cuda", dt, *case, [T - 3, 1, 1, 1], cache=op_cache(
        KVSpec(G, d, d), "cuda", dt, n_tokens=2240, max_len=2240))
    close(got[-3:], want, dt)


# --------------------------------------------------------------- recurrences
def light_case(H, d, e, T, decay):
    return {"p": rnd(T, H * (2 * d + 2 * e), seed=1, scale=1.5),
            "norm": rnd(H * e, seed=2) + 1,
            "mx": {"heads": H, "dim": d, "vdim": e, "decay": decay}}


def want_light(c, eps):
    """The oracle's mixer on h = p, its projections cutting p apart."""
    mx, n = c["mx"], c["p"].shape[1]
    a, b = mx["heads"] * mx["dim"], mx["heads"] * mx["vdim"]
    eye = torch.eye(n, dtype=torch.float64)
    w = {"q": eye[:a], "k": eye[a:2 * a], "v": eye[2 * a:2 * a + b],
         "g": eye[2 * a + b:], "norm": c["norm"],
         "o": torch.eye(b, dtype=torch.float64)}
    return O.lightning_mixer(c["p"], w, "", mx, eps)


def run_light(dev, dt, c, parts, eps, cache=None, slot=None):
    mx = c["mx"]
    cache = cache or op_cache(StateSpec(((mx["heads"], mx["vdim"],
                                          mx["dim"]),)), dev, dt)
    slot = cache.open() if slot is None else slot
    pows, dec = ops.decay_tables(mx["decay"], 64, dev)
    p, T = c["p"].to(dev, dt), c["p"].shape[0]
    got, = feed(T, parts, cache, slot, [0] * T, lambda plan, a, b: [
        ops.lightning(p[a:b].contiguous(), cache, 0, plan, pows=pows, dec=dec,
                      norm=c["norm"].to(dev, dt), eps=eps)])
    return got


STATES = [(3, 16, 24), (2, 10, 7), (1, 136, 72), (4, 64, 64), (2, 128, 128),
          (1, 1, 1), (2, 256, 200)]


@place
@cut
@pytest.mark.parametrize("shape", STATES, ids=str)
def test_lightning(dev, dt, shape, parts):
    H, d, e = shape
    c = light_case(H, d, e, 131 if parts != "tokens" else 70,
                   [0.9, 0.5, 0.999, 1.0][:H])
    close(run_light(dev, dt, c, PARTS[parts](c["p"].shape[0]), 0.02),
          want_light(c, 0.02), dt)


@place
def test_lightning_norm_spans_the_heads(dev, dt):
    """A head that is a hundred times louder quiets the others."""
    c = light_case(3, 16, 8, 40, [0.8, 0.9, 0.99])
    c["p"][:, 96:104] *= 100               # the first head's values
    c["p"] = c["p"].bfloat16().double()
    want = want_light(c, 1e-5)
    assert want[5:, 8:].abs().max() < 0.5 < want[:, :8].abs().max()
    for parts in ([40], [1] * 40):
        close(run_light(dev, dt, c, parts, 1e-5), want, dt)


def gla_case(H, d, e, T, rank=8, tau=4.0, bias=2.0, seed=0):
    a, b = H * d, H * e
    return {"q": rnd(T, a, seed=seed + 1), "k": rnd(T, a, seed=seed + 2),
            "v": rnd(T, b, seed=seed + 3), "g": rnd(T, b, seed=seed + 4),
            "u": rnd(T, rank, seed=seed + 5),
            "a2": rnd(a, rank, seed=seed + 6, scale=2 * rank ** -0.5),
            "a2.b": rnd(a, seed=seed + 7) + bias,
            "norm": rnd(e, seed=seed + 8) + 1,
            "mx": {"heads": H, "dim": d, "vdim": e, "tau": tau}}


def gla_rows(c):
    return torch.cat([c[n] for n in "qkvgu"], 1)


def want_gla(c, eps, scale=1.0):
    """The oracle's mixer on h = the rows, its projections cutting them."""
    h, w, at = gla_rows(c), {}, 0
    eye = torch.eye(h.shape[1], dtype=torch.float64)
    for n, name in zip("qkvgu", ("q", "k", "v", "g", "a1")):
        w[name] = eye[at:at + c[n].shape[1]]
        at += c[n].shape[1]
    w.update({n: c[n] for n in ("a2", "a2.b", "norm")},
             o=torch.eye(c["v"].shape[1], dtype=torch.float64))
    return O.gla_mixer(h, w, "", c["mx"], eps) * scale


def run_gla(dev, dt, c, parts, eps, scale=1.0, cache=None, slot=None):
    mx, T = c["mx"], c["q"].shape[0]
    H, d, e = mx["heads"], mx["dim"], mx["vdim"]
    cache = cache or op_cache(StateSpec(((H, e, d),)), dev, dt)
    slot = cache.open() if slot is None else slot
    x = gla_rows(c)
    x = torch.nn.functional.pad(x, (16, -x.shape[1] % 8), value=float("nan"))
    x = x.to(dev, dt)
    to = lambda t: t.to(dev, dt)

    def run(plan, a, b):
        out = torch.full((b - a, H * e + 3), 7.0, device=dev, dtype=dt)
        ops.gla(x[a:b].contiguous(), 16, out, 2, cache, 0, plan,
                rank=c["u"].shape[1], a2=to(c["a2"]), a2_b=to(c["a2.b"]),
                tau=mx["tau"], norm=to(c["norm"]), out_scale=scale, eps=eps)
        assert (out[:, :2] == 7).all() and (out[:, -1] == 7).all()
        return [out[:, 2:-1]]

    got, = feed(T, parts, cache, slot, [0] * T, run)
    return got


@place
@cut
@pytest.mark.parametrize("shape,rank", [(s, 16) for s in STATES] + [
    (s, r) for s in STATES[:2] for r in (1, 5, 40)], ids=str)
def test_gated_linear_attention(dev, dt, shape, parts, rank):
    H, d, e = shape
    c = gla_case(H, d, e, 131 if parts != "tokens" else 70, rank)
    close(run_gla(dev, dt, c, PARTS[parts](c["q"].shape[0]), 0.02, 0.7),
          want_gla(c, 0.02, 0.7), dt)


@place
@pytest.mark.parametrize("tau,bias", [(16.0, 0.0), (1.0, 0.0), (1.0, -6.0),
                                      (0.5, -40.0), (0.1, -30.0), (1.0, 30.0)])
def test_decays_from_none_to_all(dev, dt, tau, bias):
    """Channels that keep everything beside channels that forget at once:
    no power of a decay is divided out."""
    c = gla_case(2, 40, 24, 150, tau=tau, bias=bias)
    c["a2.b"][::3] = 25.0                  # these stay
    c["a2.b"][1::7] = -90.0                # these are gone in a token
    c["a2.b"] = c["a2.b"].bfloat16().double()
    want = want_gla(c, 1e-4)
    for parts in ([150], [1] * 150, cuts(150, [2, 50, 17])):
        close(run_gla(dev, dt, c, parts, 1e-4), want, dt)


@place
@pytest.mark.parametrize("gap", [1, 15, 16, 17, 48, 63, 64, 65, 140])
def test_one_token_far_back_in_a_state(dev, dt, gap):
    """A token written `gap` before the last, read by a channel that has kept
    it and faded in one that has not, across sub-tiles, tiles and portions."""
    T, H, d, e = 150, 2, 16, 16
    c = gla_case(H, d, e, T)
    at = T - 1 - gap
    for n in "qkv":
        c[n] = c[n] * (0.0 if n == "q" else 0.01)
    c["a2"] = c["a2"] * 0
    c["a2.b"] = torch.full((H * d,), 9.0, dtype=torch.float64)
    c["a2.b"][5::d] = -1.0                 # this channel fades
    q, k, v = (c[n].view(T, H, -1) for n in "qkv")
    k[at, :, 3] = k[at, :, 5] = 3.0
    v[at, 0, 2], v[at, 1, 7] = 4.0, -4.0
    q[-1, :, 3] = 1.0
    q[-2, :, 5] = 1.0
    for n in "kv":
        c[n] = c[n].bfloat16().double()
    want = want_gla(c, 1e-6)
    for parts in ([T], [T - 1, 1], [T - 2, 2], cuts(T, [37]), [at + 1, gap]):
        close(run_gla(dev, dt, c, parts, 1e-6)[-1:], want[-1:], dt)


@place
def test_long_state_does_not_drift(dev, dt):
    T = 700
    c = gla_case(1, 8, 8, T, bias=6.0, tau=16.0)
    want = want_gla(c, 1e-5)
    for parts in ([T], [100] + [1] * 600):
        close(run_gla(dev, dt, c, parts, 1e-5), want, dt)


@place
def test_states_in_a_ragged_batch(dev, dt):
    """Portions beside single tokens; slots go round; an idle row."""
    T = 90
    c = gla_case(2, 24, 16, T)
    want = want_gla(c, 0.01)
    cache = op_cache(StateSpec(((2, 16, 24),)), dev, dt)
    a, b, d = (cache.open() for _ in range(3))
    run_gla(dev, dt, {**c, **{n: c[n][:33] for n in "qkvgu"}}, [33], 0.01,
            cache=cache, slot=b)
    cache.close(a)
    a = cache.open()
    plan, _ = cache.plan([(a, [0] * T, ()), (b, [0], ()), (d, [0] * 2, ())])
    rows = gla_rows(c)
    x = torch.cat([rows[33:34], rows, rows[:2]])
    x = torch.nn.functional.pad(x, (0, -x.shape[1] % 8), value=float("nan"))
    out = torch.empty(T + 3, 32, device=dev, dtype=dt)
    to = lambda t: t.to(dev, dt)
    ops.gla(to(x), 0, out, 0, cache, 0, plan, rank=8, a2=to(c["a2"]),
            a2_b=to(c["a2.b"]), tau=4.0, norm=to(c["norm"]), out_scale=1.0,
            eps=0.01)
    close(out, torch.cat([want[33:34], want, want[:2]]), dt)


# ------------------------------------------------------------- feed-forward
@place
@pytest.mark.parametrize("T", [1, 3, 70, 400])
@pytest.mark.parametrize("E,top,ff,W", [(6, 2, 24, 32), (1, 1, 1, 8),
                                        (5, 5, 13, 27), (70, 9, 16, 48),
                                        (4, 2, 128, 64), (300, 3, 8, 16)])
def test_experts_by_token(dev, dt, T, E, top, ff, W):
    V = 29
    g = torch.Generator().manual_seed(E)
    table = torch.rand(V, E, generator=g).argsort(1)[:, :top].contiguous()
    tokens = torch.randint(0, V, (T,), generator=g)
    h = rnd(T, W, seed=1)
    gu, dn = rnd(E, 2 * ff, W, seed=2, scale=W ** -0.5), rnd(
        E, W, ff, seed=3, scale=ff ** -0.5)
    w = {"table": table}
    for e in range(E):
        w.update({f"e{e}.gate": gu[e, :ff], f"e{e}.up": gu[e, ff:],
                  f"e{e}.down": dn[e]})
    w = {k: t if k == "table" else t.bfloat16().double() for k, t in w.items()}
    parts = ops.table_moe(h.to(dev, dt), tokens.to(dev),
                          table.to(torch.int32).to(dev), gu.to(dev, dt),
                          dn.to(dev, dt))
    assert parts.y.shape == (T, top, W)
    close(parts.weights, torch.full((T, top), 1 / top, dtype=torch.float64),
          torch.float32)
    close(parts.total(), O.table_moe(h, w, "", tokens.tolist()), dt)


# ----------------------------------------------------- parts of other stacks
@place
def test_parallel_is_the_sum_of_its_sides(dev, dt):
    """Each side also stands alone, with matrices of its own."""
    from scaffold.cache import PagedStateCache
    from scaffold.models import mixers as M

    left = {"type": "window_attention", "heads": 4, "kv_heads": 2, "dim": 16,
            "vdim": 9, "scale": 0.3, "softcap": 5.0, "buckets": 9,
            "bias_max": 30, "mask": {"size": 20, "keep_first": 2}}
    right = {"type": "gla", "heads": 3, "dim": 8, "vdim": 5, "rank": 6,
             "tau": 4.0}
    W, T, eps = 40, 90, 1e-4
    torch.manual_seed(0)
    both = M.Parallel(W, {"left": left, "right": right, "left_scale": 0.6,
                          "right_scale": -1.5}, eps)
    sides = [M.WindowAttention(W, left, eps),
             M.GatedLinearAttention(W, right, eps)]
    with torch.no_grad():
        for i, side in enumerate(sides):
            own = dict(side.packed())
            for n, t in both.packed():
                if n.startswith(("left.", "right.")[i]):
                    t.copy_(rnd(*t.shape, seed=len(n) + i) * t.shape[-1] ** -0.5)
                    own[n.split(".", 1)[1]].copy_(t)
    mods = [m.to(dev, dt) for m in (both, *sides)]
    cache = PagedStateCache([m.cache_spec() for m in mods], 2, 256, 256, dev,
                            dt)
    slot, h = cache.open(), rnd(T, W, seed=3).to(dev, dt)
    with torch.no_grad():
        a, b, c = feed(T, [40, 1, 49], cache, slot, [0] * T, lambda plan, i, j: [
            m.step(h[i:j].contiguous(), plan, cache, run)
            for run, m in enumerate(mods)])
    close(a, (0.6 * b.double() - 1.5 * c.double()).cpu(), dt)
    with pytest.raises(ValueError, match="retention"):
        M.Parallel(W, {"left": left, "right": {"type": "retention"},
                       "left_scale": 1, "right_scale": 1}, eps)


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda", marks=gpu)])
@pytest.mark.parametrize("shift", [False, True])
@pytest.mark.parametrize("start", [False, True])
@pytest.mark.parametrize("loop", [False, True])
def test_every_choice_of_a_stack_alone(dev, shift, start, loop):
    """Token shift, embeddings and added loop inputs do not need each other:
    any cut gives the same logits, and a shift by nothing is no shift."""
    from scaffold.config import load_config
    from scaffold.generate import Generator
    from scaffold.models import build_model
    from tests.oracle.cases import attn, poison, ret

    def make(shift):
        cfg = load_config(None, ["model.name=lasezen", "model.vocab_size=31",
                                 "model.d_model=20", "model.norm=rms_norm",
                                 "model.post_norm=false"])
        m = cfg.model
        m.layers = [attn(), ret(ff=None)]
        m.token_shift, m.loop_add = shift, loop
        m.loop = {"start": 1, "stop": 2, "times": 3} if loop else None
        if start:
            m.sinusoid_base = 500.0
            m.bigram = {"buckets": 7, "mul_prev": 3, "mul_cur": 2}
        torch.manual_seed(1)
        model = build_model(cfg)
        with torch.no_grad():
            for n, p in model.named_parameters():
                if p.dim() > 1:
                    p.copy_(torch.randn(p.shape) * p.shape[-1] ** -0.5)
                elif n.endswith("shift"):
                    p.zero_()
        return model.to(dev).eval()

    t = torch.randint(0, 31, (70,), generator=torch.Generator().manual_seed(2))
    t = t.tolist()

    def logits(model, parts):
        cache, out, at = poison(model.new_cache(2, 256, 128)), [], 0
        s = cache.open()
        for n in parts:
            out.append(Generator(model).step(cache, [(s, t[at:at + n], range(n))]))
            at += n
        return torch.cat(out).double().cpu()

    model = make(shift)
    torch.manual_seed(1)
    plain = make(False)
    with torch.no_grad():
        sd = model.state_dict()
        plain.load_state_dict({k: v for k, v in sd.items()
                               if not k.endswith("shift")})
    want = logits(plain, [70])
    for parts in ([70], [1] * 70, cuts(70, [2, 33])):
        close(logits(model, parts), want, torch.float32, 5)
    if shift:
        with torch.no_grad():
            for b in model.blocks:
                b.shift.fill_(0.4)
        want = logits(model, [70])
        assert (want - logits(plain, [70])).abs().max() > 1e-2
        for parts in ([1] * 70, cuts(70, [2, 33])):
            close(logits(model, parts), want, torch.float32, 5)


# ------------------------------------------------------------------- checks
@gpu
def test_bindings_refuse_bad_operands():
    """What the kernels assume is checked on the host."""
    z = lambda *s: torch.zeros(*s, device="cuda")
    cache = op_cache(KVSpec(2, 16, 16), "cuda", torch.float32)
    plan, _ = cache.plan([(cache.open(), [0] * 4, ())])

    def attend(x=z(4, 128 + 64), col=0, out=z(4, 64), out_col=0, bias=z(4, 9),
               heads=4, **kw):
        ops.window_attention(
            x, col, out, out_col, cache, 0, plan, heads=heads, bias=bias,
            scale=1.0, out_scale=1.0, eps=1e-5,
            **{**dict(softcap=1.0, size=3, keep=1), **kw})

    attend()
    for bad in (dict(x=z(4, 184)), dict(col=8), dict(x=z(4, 200), col=4),
                dict(out=z(4, 63)), dict(out_col=1), dict(out=z(3, 64)),
                dict(bias=z(3, 9)), dict(heads=3), dict(size=-1),
                dict(softcap=-1.0), dict(x=z(4, 192).bfloat16()),
                dict(bias=z(4, 9).double())):
        with pytest.raises(RuntimeError):
            attend(**bad)
    sc = op_cache(StateSpec(((2, 8, 16),)), "cuda", torch.float32)
    plan, _ = sc.plan([(sc.open(), [0] * 4, ())])

    def linear(x=z(4, 104), col=0, out=z(4, 16), a2=z(32, 8), a2_b=z(32),
               norm=z(8), tau=1.0):
        ops.gla(x, col, out, 0, sc, 0, plan, rank=8, a2=a2, a2_b=a2_b, tau=tau,
                norm=norm, out_scale=1.0, eps=1e-5)

    linear()
    for bad in (dict(x=z(4, 96)), dict(col=8), dict(out=z(4, 15)),
                dict(a2=z(31, 8)), dict(a2=z(32, 16)), dict(a2_b=z(31)),
                dict(norm=z(7)), dict(tau=0.0)):
        with pytest.raises(RuntimeError):
            linear(**bad)
    st = op_cache(StateSpec(((16,),)), "cuda", torch.float32)
    plan, _ = st.plan([(st.open(), [0] * 4, ())])
    kw = dict(shift=z(16), state=st.state[0][0])
    one = torch.ones((), device="cuda")
    ops.shift_norm(z(4, 16), None, 1.0, (one,), 1e-5, plan, **kw)
    for bad in (dict(shift=z(15)), dict(state=z(3, 15)), dict(step=z(15)),
                dict(add=z(4, 15)), dict(state=None)):
        with pytest.raises(RuntimeError):
            ops.shift_norm(z(4, 16), None, 1.0, (one,), 1e-5, plan,
                           **{**kw, **bad})
    tok = torch.zeros(4, dtype=torch.int64, device="cuda")
    tab = torch.zeros(9, 2, dtype=torch.int32, device="cuda")
    ops.table_moe(z(4, 8), tok, tab, z(3, 4, 8), z(3, 8, 2))
    for bad in ((z(4, 8), tok[:3], tab, z(3, 4, 8), z(3, 8, 2)),
                (z(4, 8), tok, tab.long(), z(3, 4, 8), z(3, 8, 2)),
                (z(4, 8), tok, tab, z(3, 4, 7), z(3, 8, 2)),
                (z(4, 8), tok, tab, z(3, 4, 8), z(3, 8, 3))):
        with pytest.raises(RuntimeError):
            ops.table_moe(*bad)


def test_bucket_edges_of_the_oracle():
    """The exact half, then wider and wider spans, the last row for good."""
    rows = [O.bucket(n, 32, 128) for n in range(200)]
    assert rows[:16] == list(range(16)) and rows == sorted(rows)
    assert rows[16] == 16 and rows[127] == 31 and set(rows[128:]) == {31}
    for r in range(17, 32):                # row r begins at 16 * 8^((r-16)/16)
        first = math.ceil(16 * 8 ** ((r - 16) / 16) - 1e-9)
        assert rows[first] >= r > rows[first - 1]
