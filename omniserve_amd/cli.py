"""Command line of the engine:

    python -m omniserve_amd models                                          architectures the registry knows
    python -m omniserve_amd generate --model DIR --prompt-ids 1,2,3 [...]   token ids in, token ids out (one JSON line per prompt)
    python -m omniserve_amd trace ...                                       replay a trace (the same as bin/trace_run)
    python -m omniserve_amd build [--force]                                 compile the HIP libraries
"""
from __future__ import annotations

import argparse
import json
import sys


def _ids(text: str):
    try:
        return [int(t) for t in text.replace(" ", "").split(",") if t]
    except ValueError:
        raise argparse.ArgumentTypeError("token ids are integers with commas between them: %r" % text)


def parser() -> argparse.ArgumentParser:
    ap = argparse.ArgumentParser(prog="omniserve_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = ap.add_subparsers(dest="command", required=True)
    sub.add_parser("models")
    b = sub.add_parser("build")
    b.add_argument("--force", action="store_true")
    sub.add_parser("trace", add_help=False)
    g = sub.add_parser("generate")
    g.add_argument("--model", required=True, help="checkpoint directory (config.json and weights)")
    g.add_argument("--prompt-ids", type=_ids, action="append", default=[], help="a prompt as token ids; may be given several times")
    g.add_argument("--prompts-file", help="more prompts: one JSON list of token ids a line")
    g.add_argument("--dtype", choices=["bfloat16", "float32", "float16"], default=None, help="default: the model's own")
    g.add_argument("--max-new-tokens", type=int, default=16)
    g.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    g.add_argument("--top-k", type=int, default=0)
    g.add_argument("--top-p", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=None)
    g.add_argument("--stop-ids", type=_ids, default=[])
    g.add_argument("--cache-tokens", type=int, default=65536, help="tokens the cache pool holds")
    g.add_argument("--max-seqs", type=int, default=16, help="sequences that run at once")
    g.add_argument("--max-batch-tokens", type=int, default=8192, help="tokens of one step")
    g.add_argument("--no-graphs", action="store_true")
    return ap


def generate(a) -> int:
    import torch
    from . import models
    from .engine import Engine, SamplingParams
    prompts = list(a.prompt_ids)
    if a.prompts_file:
        with open(a.prompts_file) as f:
            prompts += [json.loads(line) for line in f if line.strip()]
    if not prompts:
        print("no prompt given (--prompt-ids or --prompts-file)", file=sys.stderr)
        return 2
    model = models.load_model(a.model, getattr(torch, a.dtype) if a.dtype else None)
    engine = Engine(model, max_tokens=a.cache_tokens, max_seqs=a.max_seqs, max_batch_tokens=a.max_batch_tokens, use_graphs=not a.no_graphs)
    params = SamplingParams(max_tokens=a.max_new_tokens, temperature=a.temperature, top_k=a.top_k, top_p=a.top_p, seed=a.seed,
                            stop_token_ids=tuple(a.stop_ids))
    for o in engine.generate(prompts, params):
        print(json.dumps({"prompt": o.prompt, "tokens": o.tokens, "finish_reason": o.finish_reason}), flush=True)
    return 0


def main(argv=None) -> int:
    argv = list(sys.argv[1:] if argv is None else argv)
    if argv[:1] == ["trace"]:
        from .trace import main as trace
        return trace(argv[1:])
    a = parser().parse_args(argv)
    if a.command == "models":
        from . import models
        print("\n".join(models.architectures()))
        return 0
    if a.command == "build":
        from . import build
        print("\n".join(build.build_all(force=a.force, verbose=True)))
        return 0
    return generate(a)
