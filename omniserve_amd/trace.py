"""Replays a trace of token ids through the engine, step by step, and writes the logits it asks for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps.jsonl

One JSON object a line on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

All entries of a step run as one batch, from the cache and state earlier steps left; a sequence is opened at its first entry and
closed after the step that lists it in "end".  A step with wanted places writes OUT/<step>.f32 ([wanted, vocab] little-endian
f32); every step prints "done <step>".  --max-tokens: the tokens (rounded up to pages per sequence) that live sequences hold at
most, which is what the cache pool is made for."""
from __future__ import annotations

import argparse
import json
import os
import sys

MAX_LIVE = 4
DTYPES = ("bfloat16", "float32")
UNSUPPORTED = 3          # exit code: the model does not run in this number format


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", choices=DTYPES, default="bfloat16")
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True)
    a = ap.parse_args(argv)

    import torch
    from . import models
    from .engine import Engine, SequenceInput
    dtype = getattr(torch, a.dtype)
    torch.backends.cuda.matmul.allow_tf32 = False
    config = models.read_config(a.model)
    cls = models.model_class(config)
    if dtype not in cls.dtypes:
        print("%s does not run in %s" % (cls.__name__, a.dtype), file=sys.stderr)
        return UNSUPPORTED
    engine = Engine(cls.from_pretrained(a.model, config, dtype), max_tokens=a.max_tokens, max_seqs=MAX_LIVE)
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        inputs = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = engine.open()
            inputs.append(SequenceInput(live[e["id"]], e["tokens"], e.get("want", ())))
        logits = engine.run(inputs)
        if logits is not None:
            logits.cpu().numpy().astype("<f4").tofile(os.path.join(a.out, "%d.f32" % step["step"]))
        else:
            torch.cuda.synchronize()
        for i in step.get("end", ()):
            engine.close(live.pop(i))
        print("done %d" % step["step"], flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
