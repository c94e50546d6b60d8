"""Replay of a token trace: given token ids go through a model step by
step, and the logits that the trace asks for are written out.  Nothing is
sampled; each step is one Generator.step over the serving cache, so it
runs the batch, pages and slots that serving would.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR
                  --max-tokens N

Standard input has one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": []}

Every entry continues its request ("id"; admitted when first seen);
"want" are places among the entry's tokens.  OUT/<step>.f32 gets the
wanted logits as little-endian float32 rows, in the order of the entries;
after every step a line `done <step>` is printed.  Requests in "end" give
their pages and slot back.
"""

from __future__ import annotations

import argparse
import json
import os
import sys

import torch

SLOTS = 4   # requests alive at a time


def replay(model, lines, out_dir: str, max_tokens: int, emit, on_layer=None
           ) -> None:
    """Run the steps of `lines` (an iterable of JSON texts); emit(step) is
    called after each, once its output is complete."""
    from .generate import Generator

    gen = Generator(model)
    if not gen.is_stack:
        raise TypeError(f"{type(model).__name__} has no ragged step")
    cache = model.new_cache(SLOTS, max_tokens, max_tokens)
    slots = {}
    for line in lines:
        if not line.strip():
            continue
        msg = json.loads(line)
        entries = []
        for e in msg["entries"]:
            if e["id"] not in slots:
                slots[e["id"]] = cache.open()
            entries.append((slots[e["id"]], e["tokens"], e.get("want", ())))
        if entries:
            logits = gen.step(cache, entries, on_layer=on_layer)
            if logits.shape[0]:
                data = logits.float().cpu().contiguous().numpy()
                path = os.path.join(out_dir, f"{msg['step']}.f32")
                with open(path, "wb") as fh:
                    fh.write(data.astype("<f4").tobytes())
        for rid in msg.get("end", ()):
            cache.close(slots.pop(rid))
        emit(msg["step"])


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"],
                    default="bfloat16")
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="cache pool size in tokens")
    ap.add_argument("--device", default="cuda", choices=["cuda", "cpu"],
                    help="cpu runs the plain test forms of the ops")
    args = ap.parse_args(argv)

    from .convert import load_model_dir
    from .ops import backend

    if args.device == "cuda":
        if not torch.cuda.is_available():
            print("trace_run: no GPU", file=sys.stderr)
            return 2
        backend.ensure_lm_ext()
    torch.backends.cuda.matmul.allow_tf32 = False
    model = load_model_dir(args.model, getattr(torch, args.dtype),
                           args.device)
    os.makedirs(args.out, exist_ok=True)
    replay(model, sys.stdin, args.out, args.max_tokens,
           lambda step: print(f"done {step}", flush=True))
    return 0


if __name__ == "__main__":
    sys.exit(main())
