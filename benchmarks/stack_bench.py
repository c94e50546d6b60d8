"""Prefill and decode throughput of mixer-stack designs, each beside the
model it is closest to (random weights): Lasezen beside Llama at equal
width, heads, feed-forward width and depth; Nekozen beside Lasezen at
equal width, heads and depth, its feed-forwards two thirds as wide because
they have three matrices; Babodra beside Lasezen at equal width, heads and
depth, with as many feed-forward weights active per token; Tilivik beside
Babodra at equal width, heads, depth, experts and active feed-forward weights.

Run through bench.py: `python bench.py --model lasezen|nekozen|babodra|tilivik
[--steps K] [--warmup W]`.  One JSON line per size and phase; decode steps are
hipGraph replays of the serving step for all models.
"""

from __future__ import annotations

import json
import statistics
import time

import torch

from scaffold.config import TrainConfig, load_config
from scaffold.generate import Generator
from scaffold.models import build_model

# width, heads, kv heads, head dim, ff, chunk, layers, vocab
SIZES = {
    "w2048": dict(width=2048, heads=16, kv=4, dim=128, ff=8192, chunk=1024,
                  layers=8, vocab=32768),
    "w4096": dict(width=4096, heads=32, kv=8, dim=128, ff=14336, chunk=2048,
                  layers=8, vocab=32768),
}
MAX_LEN = 8192 + 512
# what a benchmark of a design measures
BESIDE = {"lasezen": ("lasezen", "llama"), "nekozen": ("nekozen", "lasezen"),
          "babodra": ("babodra", "lasezen"),
          "tilivik": ("tilivik", "lasezen", "babodra")}


def lasezen_config(s: dict) -> TrainConfig:
    """Every fourth layer retention, the others chunk attention, all with
    a feed-forward (Llama has one in every layer)."""
    H = s["heads"]
    ff = {"kind": "dense", "ff": s["ff"]}
    ret = {"type": "retention", "mlp": ff, "mixer": {
        "heads": H, "dim": s["dim"], "vdim": s["dim"],
        "rot": {"base": 10000.0, "dims": s["dim"]},
        "decay": [1 - 2.0 ** (-5 - 3 * h / H) for h in range(H)]}}
    att = {"type": "attention", "mlp": ff, "mixer": {
        "heads": H, "kv_heads": s["kv"], "dim": s["dim"], "vdim": s["dim"],
        "mask": {"size": s["chunk"]}, "scale": s["dim"] ** -0.5}}
    cfg = load_config(None, ["model.name=lasezen",
                             f"model.vocab_size={s['vocab']}",
                             f"model.d_model={s['width']}",
                             f"model.max_seq_len={MAX_LEN}"])
    cfg.model.layers = [ret if i % 4 == 0 else att
                        for i in range(s["layers"])]
    return cfg


def nekozen_config(s: dict) -> TrainConfig:
    """Of four layers two latent attention, one Mamba-2, one mLSTM; the
    second half of the stack is the loop's span, run once."""
    W, H = s["width"], s["heads"]
    ff = {"kind": "gated", "ff": s["ff"] * 2 // 3 // 256 * 256}
    att = {"type": "latent_attention", "mlp": ff, "mixer": {
        "heads": H, "dim": s["dim"], "rot_dim": s["dim"] // 2,
        "vdim": s["dim"], "kv_rank": 512, "q_rank": 3 * W // 8,
        "mask": {"size": s["chunk"]}, "scale": (1.5 * s["dim"]) ** -0.5,
        "rot": {"base": 10000.0, "dims": s["dim"] // 2,
                "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0,
                            "slow": 1.0}}}}
    ssm = {"type": "mamba2", "mlp": ff, "mixer": {
        "heads": W // 32, "vdim": 64, "state": 128, "groups": 8, "conv": 4,
        "norm_groups": 8}}
    mem = {"type": "mlstm", "mlp": ff, "mixer": {
        "heads": W // 256, "dim": 128, "vdim": 256, "gate_cap": 15.0}}
    cfg = load_config(None, ["model.name=nekozen",
                             f"model.vocab_size={s['vocab']}",
                             f"model.d_model={W}",
                             f"model.max_seq_len={MAX_LEN}",
                             "model.logit_softcap=30"])
    n = s["layers"]
    cfg.model.layers = [(mem, att, ssm, att)[i % 4] for i in range(n)]
    cfg.model.loop = {"start": n // 2, "stop": n, "times": 1}
    return cfg


def babodra_config(s: dict) -> TrainConfig:
    """One dense layer, the others 32 experts in 4 groups, 4 of 2 groups
    chosen, and a shared one: 5 small experts of three matrices have the
    active weights of Lasezen's two."""
    ff = s["ff"] * 2 // 15 // 64 * 64
    mix = {"heads": s["heads"], "kv_heads": s["kv"], "dim": s["dim"],
           "vdim": s["dim"], "scale": s["dim"] ** -0.5,
           "q_temp": {"coef": 0.1, "every": 2048}}
    moe = {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": ff},
           "router": {"experts": 32, "top": 4, "scale": 1.0,
                      "groups": {"count": 4, "keep": 2}}}
    dense = {"kind": "clamped", "ff": s["ff"] * 2 // 3 // 256 * 256,
             "limit": 7.0}
    cfg = load_config(None, ["model.name=babodra",
                             f"model.vocab_size={s['vocab']}",
                             f"model.d_model={s['width']}",
                             f"model.positions={MAX_LEN}"])
    cfg.model.layers = [{"type": "tied_attention", "mixer": mix,
                         "mlp": moe if i else dense}
                        for i in range(s["layers"])]
    return cfg


def tilivik_config(s: dict) -> TrainConfig:
    """Every fourth layer lightning, the others window attention beside gated
    linear attention with a quarter of its heads; in every layer 32 experts of
    which a token id takes 5, as wide as Babodra's.  The second half of the
    stack is the loop's span, run once."""
    H, n = s["heads"], s["layers"]
    moe = {"kind": "table_moe", "router": {"experts": 32, "top": 5},
           "expert": {"ff": s["ff"] * 2 // 15 // 64 * 64}}
    light = {"type": "lightning", "mlp": moe, "mixer": {
        "heads": H, "dim": s["dim"], "vdim": s["dim"],
        "decay": [1 - 2.0 ** (-5 - 3 * h / H) for h in range(H)]}}
    both = {"type": "parallel", "mlp": moe, "mixer": {
        "left": {"type": "window_attention", "heads": H, "kv_heads": s["kv"],
                 "dim": s["dim"], "vdim": s["dim"], "buckets": 32,
                 "bias_max": 128, "scale": s["dim"] ** -0.5, "softcap": 50.0,
                 "mask": {"size": s["chunk"], "keep_first": 4}},
        "right": {"type": "gla", "heads": H // 4, "dim": s["dim"],
                  "vdim": s["dim"], "rank": 16, "tau": 16.0},
        "left_scale": 0.7, "right_scale": 1.0}}
    cfg = load_config(None, ["model.name=tilivik",
                             f"model.vocab_size={s['vocab']}",
                             f"model.d_model={s['width']}",
                             f"model.max_seq_len={MAX_LEN}"])
    cfg.model.bigram = {"buckets": s["vocab"], "mul_prev": 8191,
                        "mul_cur": 127}
    cfg.model.layers = [both if i % 4 else light for i in range(n)]
    cfg.model.loop = {"start": n // 2, "stop": n, "times": 1}
    return cfg


def llama_config(s: dict) -> TrainConfig:
    return load_config(None, [
        "model.name=llama", f"model.vocab_size={s['vocab']}",
        f"model.d_model={s['width']}", f"model.n_layers={s['layers']}",
        f"model.n_heads={s['heads']}", f"model.n_kv_heads={s['kv']}",
        f"model.d_ff={s['ff']}", f"model.max_seq_len={MAX_LEN}"])


def build(name: str, s: dict, dtype=torch.bfloat16):
    torch.manual_seed(0)
    cfg = {"lasezen": lasezen_config, "nekozen": nekozen_config,
           "babodra": babodra_config, "tilivik": tilivik_config,
           "llama": llama_config}[name](s)
    with torch.device("cuda"):       # random init on the GPU
        model = build_model(cfg)
    # llama builds its rotary tables on the host: move what is left
    return model.to("cuda", dtype).eval()


def _time(fn, steps, warmup):
    """Median milliseconds of fn() over `steps` timed calls."""
    for _ in range(warmup):
        fn()
    marks = [torch.cuda.Event(enable_timing=True) for _ in range(steps + 1)]
    torch.cuda.synchronize()
    marks[0].record()
    for i in range(steps):
        fn()
        marks[i + 1].record()
    torch.cuda.synchronize()
    return statistics.median(marks[i].elapsed_time(marks[i + 1])
                             for i in range(steps))


@torch.no_grad()
def prefill_ms(gen, B, S, steps, warmup):
    """One forward pass over B prompts of S tokens, last logits."""
    dev = next(gen.m.parameters()).device
    toks = torch.randint(0, gen.m.lm_head.weight.shape[0], (B, S), device=dev)
    cache = gen.new_cache(B, S)

    def run():
        if gen.is_stack:
            cache.lens = [0] * B
        else:
            cache.len = 0
        gen._forward_tokens(toks, cache, 0)

    return _time(run, steps, warmup)


@torch.no_grad()
def decode_ms(gen, B, ctx, steps, warmup):
    """One graph-replayed decode step of B rows at positions ctx...
    (keys and values as the cache starts; their values do not matter)."""
    dev = next(gen.m.parameters()).device
    n = steps + warmup + 4
    cache = gen.new_cache(B, ctx + n)
    # unequal tokens: equal ones would all choose the same experts
    cur = torch.arange(1, B + 1, device=dev).view(B, 1) * 97
    pos = torch.tensor([ctx], dtype=torch.int64, device=dev)
    out = torch.zeros(B, ctx + n + 1, dtype=torch.int64, device=dev)
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        for _ in range(2):
            gen._decode_step_static(cur, cache, pos, out)
    torch.cuda.current_stream().wait_stream(side)
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        gen._decode_step_static(cur, cache, pos, out)
    return _time(g.replay, steps, warmup)


def run(steps: int, warmup: int, sizes=None, models=BESIDE["lasezen"],
        prefill=((1, 8192), (8, 1024)), decode=((1, 4000), (8, 4000), (64, 4000)),
        emit=lambda r: print(json.dumps(r), flush=True)):
    for size in sizes or SIZES:
        s = SIZES[size]
        for name in models:
            t0 = time.time()
            gen = Generator(build(name, s))
            n_par = sum(p.numel() for p in gen.m.parameters())
            base = {"model": name, "size": size, "params_m": round(n_par / 1e6),
                    "dtype": "bf16", "data": "synthetic", "n_gpus": 1,
                    "steps": steps, "warmup": warmup}
            for B, S in prefill:
                ms = prefill_ms(gen, B, S, steps, warmup)
                emit({"metric": "prefill_tokens_per_sec",
                      "value": round(B * S / ms * 1e3), "unit": "tokens/s",
                      "ms_per_step": round(ms, 3), "batch": B, "seq_len": S,
                      **base})
            for B, ctx in decode:
                ms = decode_ms(gen, B, ctx, steps, warmup)
                emit({"metric": "decode_tokens_per_sec",
                      "value": round(B / ms * 1e3), "unit": "tokens/s",
                      "ms_per_step": round(ms, 4), "batch": B,
                      "context": ctx, **base})
            del gen
            torch.cuda.empty_cache()
            print(f"# {size} {name}: {time.time() - t0:.0f} s", flush=True)
