"""Small random mixer-stack models and plans for the tests."""

import random

import torch

from scaffold.cache import KVSpec, PagedStateCache, StateSpec, TiedSpec
from scaffold.config import load_config
from scaffold.convert import load_stack
from scaffold.models import build_model
from tests.oracle import babodra, lasezen, nekozen, tilivik

ORACLES = {"Lasezen": lasezen, "Nekozen": nekozen, "Babodra": babodra,
           "Tilivik": tilivik}


def attn(heads=4, kv=2, dim=16, vdim=16, size=24, scale=0.3, ff=40):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim,
                      "vdim": vdim, "mask": {"size": size}, "scale": scale},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def ret(heads=3, dim=16, vdim=24, rot=16, base=1000.0, decay=None, ff=40):
    return {"type": "retention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "rot": {"dims": rot, "base": base},
                      "decay": decay or [0.98, 0.9, 0.999, 0.7][:heads]},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width=32, vocab=61, loop=None, mult=0.5, eps=1e-5):
    return {"architecture": "Lasezen", "layers": layers, "width": width,
            "vocab": vocab, "norm": {"eps": eps}, "residual_mult": mult,
            "loop": loop or {"start": 0, "stop": len(layers), "times": 1}}


# name -> configuration; each makes some part matter that others leave idle
CONFIGS = {
    "plain": config([ret(), attn()]),
    "looped": config([attn(size=17, ff=None), ret(ff=None), attn(kv=1),
                      ret(heads=1, dim=12, vdim=8, rot=6, decay=[0.95])],
                     loop={"start": 1, "stop": 3, "times": 3}, mult=0.8),
    "odd": config([ret(heads=2, dim=10, vdim=7, rot=4, base=50.0),
                   attn(heads=3, kv=3, dim=9, vdim=5, size=5, ff=21)],
                  width=27, vocab=33, eps=0.05),
    "wide": config([attn(heads=6, kv=2, dim=72, vdim=136, size=100),
                    ret(heads=2, dim=72, vdim=136, rot=64)],
                   width=48, mult=1.0),
    "ones": config([attn(heads=1, kv=1, dim=32, vdim=32, size=1, scale=1.0),
                    ret(heads=1, dim=32, vdim=32, rot=2, decay=[1.0]),
                    attn(heads=2, kv=1, size=4096, scale=0.2)], mult=1.0),
}


def latent(heads=3, dim=24, rot=8, vdim=16, rank=32, q_rank=24, size=20,
           scale=0.25, base=500.0, yarn=None, ff=40):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot,
                      "vdim": vdim, "kv_rank": rank, "q_rank": q_rank,
                      "mask": {"size": size}, "scale": scale,
                      "rot": {"dims": rot, "base": base,
                              "scaling": yarn or YARN}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def mamba(heads=4, vdim=16, state=24, groups=2, conv=4, parts=2, ff=40):
    return {"type": "mamba2",
            "mixer": {"heads": heads, "vdim": vdim, "state": state,
                      "groups": groups, "conv": conv, "norm_groups": parts},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mem(heads=3, dim=16, vdim=24, cap=6.0, ff=40):
    return {"type": "mlstm",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "gate_cap": cap},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def nekozen_config(layers, width=32, vocab=61, loop=None, cap=9.0, eps=1e-5):
    return {"architecture": "Nekozen", "layers": layers, "width": width,
            "vocab": vocab, "norm": {"eps": eps}, "logit_softcap": cap,
            "loop": loop or {"start": 0, "stop": len(layers), "times": 1}}


NEKOZEN = {
    "neko-plain": nekozen_config([latent(size=33), mamba(), mem()]),
    "neko-looped": nekozen_config(
        [mem(), latent(size=17, ff=None), mamba(ff=None, parts=4),
         mem(heads=2, dim=12, vdim=40), latent(heads=2, size=70)],
        loop={"start": 1, "stop": 4, "times": 3}, cap=4.0),
    "neko-odd": nekozen_config(
        [mamba(heads=6, vdim=7, state=10, groups=3, conv=3, parts=2),
         latent(heads=5, dim=9, rot=6, vdim=5, rank=21, q_rank=13, size=5,
                ff=21),
         mem(heads=2, dim=9, vdim=5, cap=2.0)],
        width=27, vocab=33, eps=0.05, loop={"start": 1, "stop": 2, "times": 2}),
    "neko-wide": nekozen_config(
        [latent(heads=17, dim=72, rot=64, vdim=72, rank=136, q_rank=40,
                size=100),
         mamba(heads=2, vdim=136, state=72, groups=1, conv=2, parts=1),
         mem(heads=1, dim=72, vdim=136)], width=48),
    "neko-ones": nekozen_config(
        [mamba(heads=1, vdim=32, state=32, groups=1, conv=1, parts=1),
         latent(heads=1, dim=32, rot=2, vdim=32, rank=1, q_rank=1, size=1,
                scale=1.0),
         latent(heads=2, size=4096),
         mem(heads=1, dim=1, vdim=1, cap=30.0),
         mamba(heads=3, vdim=8, state=1, groups=3, conv=5, parts=3)],
        loop={"start": 2, "stop": 5, "times": 1}),
}
CONFIGS.update(NEKOZEN)


def tied(heads=4, kv=2, dim=16, scale=0.35, coef=0.7, every=20, mlp=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim,
                      "scale": scale, "q_temp": {"coef": coef, "every": every}},
            "mlp": mlp}


def clamped(ff=40, limit=0.9):
    return {"kind": "dense", "ff": ff, "limit": limit}


def routed(experts=8, top=3, groups=4, keep=2, ff=24, shared=40, scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "top": top, "scale": scale,
                       "groups": {"count": groups, "keep": keep}}}


def babodra_config(layers, width=32, vocab=61, positions=300, eps=1e-5):
    return {"architecture": "Babodra", "layers": layers, "width": width,
            "vocab": vocab, "norm": {"eps": eps}, "max_positions": positions}


BABODRA = {
    "bab-plain": babodra_config(
        [tied(mlp=clamped()), tied(kv=1, mlp=routed()), tied(kv=4)]),
    "bab-odd": babodra_config(
        [tied(heads=3, kv=3, dim=9, every=7,
              mlp=routed(5, 3, 5, 4, ff=13, shared=9)),
         tied(heads=2, kv=1, dim=5), tied(heads=5, kv=1, dim=7, coef=-0.1,
                                          mlp=clamped(21, 2.5))],
        width=27, vocab=33, positions=150, eps=0.05),
    "bab-wide": babodra_config(
        [tied(heads=6, kv=2, dim=72, scale=0.1, every=64,
              mlp=routed(70, 9, 7, 2, ff=16, shared=72)),
         tied(heads=8, kv=1, dim=136, scale=0.08, mlp=clamped(72, 0.3))],
        width=48),
    "bab-even": babodra_config(
        [tied(heads=2, kv=2, dim=64, scale=0.15, mlp=clamped(128, 1.1)),
         tied(heads=2, kv=1, dim=128, scale=0.1, every=33,
              mlp=routed(4, 2, 2, 2, ff=64, shared=128)),
         tied(mlp=routed(6, 2, 2, 1, ff=128, shared=64, scale=0.8))],
        width=64),
    "bab-ones": babodra_config(
        [tied(heads=1, kv=1, dim=32, scale=1.0, coef=0.2, every=1,
              mlp=routed(1, 1, 1, 1, ff=1, shared=1, scale=1.0)),
         tied(heads=1, kv=1, dim=1, coef=0.0, every=4096,
              mlp=routed(3, 3, 1, 1))]),
}
CONFIGS.update(BABODRA)


def table_ff(experts=6, top=2, ff=24):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top}}


def light(heads=3, dim=16, vdim=24, decay=None, mlp=None):
    return {"type": "lightning", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim,
        "decay": decay or [0.97, 0.6, 0.999, 0.85][:heads]}}


def window(heads=4, kv=2, dim=16, vdim=24, size=21, keep=3, far=50, scale=0.3,
           cap=6.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "bias_max": far, "mask": {"size": size, "keep_first": keep},
            "scale": scale, "softcap": cap}


def chan(heads=3, dim=24, vdim=16, tau=4.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def par(left=None, right=None, ls=0.7, rs=1.3, mlp=None):
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": left or window(), "right": right or chan(), "left_scale": ls,
        "right_scale": rs}}


def tilivik_config(layers, width=32, vocab=61, loop=None, eps=1e-5,
                   buckets=97, muls=(31, 11), rel=14, rank=8):
    """rel, rank: sizes that only the tensors' shapes tell."""
    return {"architecture": "Tilivik", "layers": layers, "width": width,
            "vocab": vocab, "norm": {"eps": eps}, "loop": loop,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": muls[0],
                                     "mul_cur": muls[1]}},
            "_rel": rel, "_rank": rank}


TILIVIK = {
    "tili-plain": tilivik_config([light(mlp=table_ff()),
                                  par(mlp=table_ff(5, 3))]),
    "tili-looped": tilivik_config(
        [light(heads=2), par(window(kv=1, size=33, keep=0), mlp=table_ff()),
         light(heads=4, dim=12, vdim=8, mlp=table_ff(4, 1)),
         par(window(heads=2, kv=2, size=70, keep=66), chan(tau=1.0))],
        loop={"start": 1, "stop": 3, "times": 3}),
    "tili-odd": tilivik_config(
        [par(window(heads=3, kv=3, dim=9, vdim=5, size=5, keep=1, far=9),
             chan(heads=2, dim=10, vdim=7, tau=0.7), mlp=table_ff(5, 3, 13)),
         light(heads=3, dim=5, vdim=7, mlp=table_ff(3, 3, 9)),
         par(window(heads=5, kv=1, dim=7, vdim=9, size=64, keep=64),
             chan(heads=5, dim=9, vdim=3))],
        width=27, vocab=33, eps=0.05, buckets=13, muls=(5, 3), rel=7, rank=5,
        loop={"start": 0, "stop": 2, "times": 2}),
    "tili-wide": tilivik_config(
        [par(window(heads=6, kv=2, dim=72, vdim=136, size=100, keep=70,
                    scale=0.1, far=128),
             chan(heads=2, dim=136, vdim=72), mlp=table_ff(70, 9, 16)),
         light(heads=2, dim=72, vdim=136)],
        width=48, rel=32, rank=16, loop={"start": 1, "stop": 2, "times": 2}),
    "tili-even": tilivik_config(
        [par(window(heads=4, kv=2, dim=64, vdim=64, size=48, keep=5,
                    scale=0.125, far=128, cap=30.0),
             chan(heads=2, dim=64, vdim=128, tau=16.0),
             mlp=table_ff(8, 2, 64)),
         light(heads=2, dim=64, vdim=64, mlp=table_ff(4, 2, 128)),
         par(window(heads=4, kv=1, dim=128, vdim=64, size=130, keep=8,
                    scale=0.1), chan(heads=1, dim=128, vdim=64, tau=8.0))],
        width=64, rel=32, rank=16),
    "tili-ones": tilivik_config(
        [light(heads=1, dim=1, vdim=1, decay=[1.0], mlp=table_ff(1, 1, 1)),
         par(window(heads=1, kv=1, dim=1, vdim=1, size=1, keep=0, far=2,
                    scale=1.0, cap=1.0),
             chan(heads=1, dim=1, vdim=1, tau=1.0), ls=1.0, rs=1.0),
         par(window(heads=2, kv=1, size=4096, keep=1, far=4096),
             chan(heads=1, dim=32, vdim=32))],
        buckets=1, muls=(0, 1), rel=2, rank=1,
        loop={"start": 1, "stop": 3, "times": 1}),
}
CONFIGS.update(TILIVIK)


def oracle(cfg):
    return ORACLES[cfg["architecture"]]


def nekozen_weights(cfg, seed=0):
    """As weights(): no gate, decay, bias or norm is near what would leave
    it out."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, around=1.0, spread=0.4):
        w[name] = around + spread * torch.randn(n, generator=g)

    def norm(name):
        vec(name, W)
        vec(name + ".b", W, 0.0, 0.3)
        w[name + ".alpha"] = (0.4 + 0.4 * torch.rand(1, generator=g))[0]

    w["embed"] = torch.randn(V, W, generator=g)
    if cfg["loop"]:
        mat("loop.in", W, 2 * W, 1.4)
        w["loop.step"] = torch.randn(cfg["loop"]["times"], W, generator=g) * 0.5
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        for n in ("norm1", "norm2") if L["mlp"] else ("norm1",):
            norm(p + n)
        p += "mix."
        H, e = mx["heads"], mx["vdim"]
        if L["type"] == "latent_attention":
            d, r, k, c = (mx[n] for n in ("dim", "rot_dim", "kv_rank",
                                          "q_rank"))
            mat(p + "dq", c, W)
            vec(p + "dq.norm", c, 1.5)
            mat(p + "uq", H * (d + r), c, 1.5)
            mat(p + "dkv", k + r, W)
            vec(p + "dkv.norm", k)
            mat(p + "uk", H * d, k)
            mat(p + "uv", H * e, k)
            mat(p + "g", H, W, 2.0)
        elif L["type"] == "mamba2":
            G, n = mx["groups"], mx["state"]
            ch = H * e + 2 * G * n
            mat(p + "in", H * e + ch + H, W, 1.5)
            mat(p + "conv", ch, mx["conv"], 1.5)
            vec(p + "conv.b", ch, 0.0)
            vec(p + "dt_bias", H, -1.5, 1.0)
            vec(p + "A_log", H, 0.0, 1.0)
            vec(p + "D", H)
            vec(p + "norm", H * e)
        else:
            d = mx["dim"]
            mat(p + "q", H * d, W)
            mat(p + "k", H * d, W)
            mat(p + "v", H * e, W)
            mat(p + "g", H * e, W, 2.0)
            mat(p + "i", H, W, 3.0)
            vec(p + "i.b", H, 0.0, 1.0)
            mat(p + "f", H, W, 2.0)
            vec(p + "f.b", H, 3.0, 1.0)
            vec(p + "norm", H * e)
        mat(p + "o", W, H * e)
        if L["mlp"]:
            for n in ("gate", "up"):
                mat(f"l{i}.mlp.{n}", L["mlp"]["ff"], W, 1.5)
            mat(f"l{i}.mlp.down", W, L["mlp"]["ff"])
    norm("final.norm")
    mat("head", V, W, 3.0)
    return {k: v.bfloat16().float() for k, v in w.items()}


def babodra_weights(cfg, seed=0):
    """As weights(): scores, gates and clamps all at work."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, around=1.0, spread=0.4):
        w[name] = around + spread * torch.randn(n, generator=g)

    def expert(p, ff):
        mat(p + "gate", ff, W, 1.2)
        mat(p + "up", ff, W, 1.2)
        mat(p + "down", W, ff)

    w["embed"] = torch.randn(V, W, generator=g)
    w["pos"] = torch.randn(cfg["max_positions"], W, generator=g) * 0.5
    for i, L in enumerate(cfg["layers"]):
        p, mx, ff = f"l{i}.", L["mixer"], L["mlp"]
        for n in ("norm1", "norm2") if ff else ("norm1",):
            vec(p + n, W, 0.8)
        a, b = mx["heads"] * mx["dim"], mx["kv_heads"] * mx["dim"]
        for n, rows in (("q", a), ("k", b)):
            mat(f"{p}mix.{n}", rows, W)
            vec(f"{p}mix.{n}.b", rows, 0.0, 0.5)
            vec(f"{p}mix.{n}.norm", rows, 1.3)
        mat(p + "mix.g", a, W, 2.0)
        mat(p + "mix.o", W, a)
        if ff and ff["kind"] == "dense":
            expert(p + "mlp.", ff["ff"])
        elif ff:
            E = ff["router"]["experts"]
            for e in range(E):
                expert(f"{p}mlp.e{e}.", ff["expert"]["ff"])
            mat(p + "mlp.router", E, W, 0.9)
            expert(p + "mlp.shared.", ff["shared"]["ff"])
            mat(p + "mlp.shared.sg", 1, W, 1.5)
    vec("final.norm", W)
    mat("head", V, W, 3.0)
    return {k: v.bfloat16().float() for k, v in w.items()}


def tilivik_weights(cfg, seed=0):
    """As weights(): no shift, gate, bias, cap or decay is near what would
    leave it out."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, around=1.0, spread=0.4):
        w[name] = around + spread * torch.randn(n, generator=g)

    def num(name):
        w[name] = 0.8 + 0.4 * torch.rand((), generator=g)

    mat("embed", V, W, W ** 0.5)
    mat("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, W, W ** 0.5)
    if cfg["loop"]:
        mat("loop.step", cfg["loop"]["times"], W, W ** 0.5)
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        for n in ("norm1", "norm2") if L["mlp"] else ("norm1",):
            num(p + n)
        vec(p + "shift", W, 0.4, 0.3)
        if L["type"] == "lightning":
            a, b = mx["heads"] * mx["dim"], mx["heads"] * mx["vdim"]
            for n, rows in (("q", a), ("k", a), ("v", b), ("g", b)):
                mat(f"{p}mix.{n}", rows, W, 1.5)
            mat(p + "mix.o", W, b)
            vec(p + "mix.norm", b)
        else:
            m, q = mx["left"], p + "mix.left."
            mat(q + "q", m["heads"] * m["dim"], W, 2.0)
            mat(q + "k", m["kv_heads"] * m["dim"], W, 2.0)
            mat(q + "v", m["kv_heads"] * m["vdim"], W)
            mat(q + "g", m["heads"] * m["vdim"], W, 2.0)
            mat(q + "o", W, m["heads"] * m["vdim"])
            w[q + "rel"] = torch.randn(cfg["_rel"], m["heads"], generator=g)
            m, q = mx["right"], p + "mix.right."
            a, b = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, rows in (("q", a), ("k", a), ("v", b), ("g", b)):
                mat(q + n, rows, W, 1.5)
            mat(q + "a1", cfg["_rank"], W)
            mat(q + "a2", a, cfg["_rank"], 2.0)
            vec(q + "a2.b", a, 2.0, 1.5)
            mat(q + "o", W, b)
            vec(q + "norm", m["vdim"])
        if L["mlp"]:
            E, top = (L["mlp"]["router"][n] for n in ("experts", "top"))
            ff = L["mlp"]["expert"]["ff"]
            for e in range(E):
                mat(f"{p}mlp.e{e}.gate", ff, W, 1.5)
                mat(f"{p}mlp.e{e}.up", ff, W, 1.5)
                mat(f"{p}mlp.e{e}.down", W, ff, 1.5)
            w[p + "mlp.table"] = torch.rand(V, E, generator=g).argsort(
                1)[:, :top].to(torch.int32).contiguous()
    num("final.norm")
    mat("head", V, W, 3.0)
    return {k: v.bfloat16().float() if v.is_floating_point() else v
            for k, v in w.items()}


def weights(cfg, seed=0):
    """Random checkpoint (bfloat16-representable float32 tensors), scaled
    so that scores, sinks and norms are far from trivial."""
    if cfg["architecture"] == "Babodra":
        return babodra_weights(cfg, seed)
    if cfg["architecture"] == "Nekozen":
        return nekozen_weights(cfg, seed)
    if cfg["architecture"] == "Tilivik":
        return tilivik_weights(cfg, seed)
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, around=1.0, spread=0.4):
        w[name] = around + spread * torch.randn(n, generator=g)

    def norm(name):
        vec(name, W)
        vec(name + ".b", W, 0.0, 0.3)

    w["embed"] = torch.randn(V, W, generator=g)
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if L["mlp"] else ()):
            norm(p + n)
        H, d, e = mx["heads"], mx["dim"], mx["vdim"]
        if L["type"] == "attention":
            G = mx["kv_heads"]
            mat(p + "mix.q", H * d, W)
            mat(p + "mix.k", G * d, W)
            mat(p + "mix.v", G * e, W)
            vec(p + "mix.q.norm", d, 1.5)
            vec(p + "mix.k.norm", d, 1.5)
            vec(p + "mix.sink", H, 1.0, 1.0)
        else:
            mat(p + "mix.q", H * d, W)
            mat(p + "mix.k", H * d, W)
            mat(p + "mix.v", H * e, W)
            mat(p + "mix.g", H * e, W, 2.0)
        mat(p + "mix.o", W, H * e)
        if L["mlp"]:
            mat(p + "mlp.up", L["mlp"]["ff"], W, 1.5)
            mat(p + "mlp.down", W, L["mlp"]["ff"])
    norm("final.norm")
    mat("head", V, W, 2.0)
    return {k: v.bfloat16().float() for k, v in w.items()}


def build(cfg, w, device="cpu", dtype=torch.float32, max_len=512):
    from scaffold import config as C

    tc = load_config(None, [f"model.max_seq_len={max_len}"])
    shapes = {k: tuple(v.shape) for k, v in w.items()}
    for k, v in C.ARCHITECTURES[cfg["architecture"]](cfg, shapes).items():
        setattr(tc.model, k, v)
    m = build_model(tc)
    load_stack(m, w)
    return m.to(device, dtype).eval()


def tokens(cfg, n, seed=1):
    r = random.Random(seed)
    return [r.randrange(cfg["vocab"]) for _ in range(n)]


def poison(cache):
    """Fill every page and state with NaN: whatever is read before it is
    written shows in the result."""
    for t in cache.k + cache.v + [t for s in cache.state for t in s or ()]:
        if t is not None:
            t.fill_(float("nan") if t.is_floating_point() else -10**15)
    return cache


def op_cache(spec, device, dtype, slots=3, n_tokens=1024, max_len=1024):
    return poison(PagedStateCache([spec], slots, n_tokens, max_len, device,
                                  dtype))


def cuts(n, sizes):
    """Portion lengths covering n tokens, cycling through `sizes`."""
    out, i = [], 0
    while n > 0:
        c = min(n, sizes[i % len(sizes)])
        out.append(c)
        n -= c
        i += 1
    return out


__all__ = ["attn", "ret", "latent", "mamba", "mem", "config",
           "nekozen_config", "tied", "clamped", "routed", "babodra_config",
           "light", "window", "chan", "par", "table_ff", "tilivik_config",
           "CONFIGS", "NEKOZEN", "BABODRA", "TILIVIK", "oracle", "weights", "build",
           "tokens", "poison", "op_cache", "cuts", "KVSpec", "StateSpec",
           "TiedSpec"]
