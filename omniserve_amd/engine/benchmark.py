"""Prefill and decode throughput of an engine model at sizes that resemble a real model's layers (random weights; `bench.py
--design`): Bobavik beside the W4A8KV4 Llama runner with the same width, heads, number of layers and active feed-forward channels,
Bagedra beside a Bobavik of the same width, heads and feed-forward (one expert, always chosen) with softmax attention in place of the
latent one and decayed linear attention in place of the other recurrences."""
from __future__ import annotations

import gc
import sys
import time

import torch

from ..models import model_class
from ..runtime import DecodeRunner, LlamaConfig
from . import Engine, SequenceInput

# width, heads, kv heads, head size, experts, top, expert ff, shared ff (top * ff + shared = the Llama's feed-forward), window
SIZES = {
    "4096": dict(width=4096, heads=32, kv_heads=8, dim=128, experts=32, top=6, ff=1792, shared=3584, window=4096, vocab=128256),
    "2048": dict(width=2048, heads=16, kv_heads=4, dim=128, experts=64, top=8, ff=640, shared=1024, window=1024, vocab=32000),
}
LAYERS = ("attention", "lightning", "lightning", "attention", "lightning", "lightning", "attention", "lightning")

# width = heads * dim; key heads of the delta rule, latent and turned key part of latent attention, rank of the decays' projection
BAGEDRA_SIZES = {
    "4096": dict(width=4096, heads=32, kv_heads=16, dim=128, kv_rank=512, rot_dim=64, rank=16, conv=4, ff=14336, vocab=128256),
    "2048": dict(width=2048, heads=16, kv_heads=8, dim=128, kv_rank=256, rot_dim=64, rank=16, conv=4, ff=6144, vocab=32000),
}
BAGEDRA_LAYERS = ("gla", "delta", "latent_attention", "gla", "delta", "latent_attention", "gla", "delta")


def bagedra_config(s: dict) -> dict:
    soft = {"heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "kv_rank": s["kv_rank"], "rot_dim": s["rot_dim"],
            "rot": {"dims": s["rot_dim"], "base": 500000.0}, "scale": (s["dim"] + s["rot_dim"]) ** -0.5}
    mixers = {"latent_attention": soft, "gla": {"heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "tau": 16.0},
              "delta": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "conv": s["conv"]}}
    return {"architecture": "Bagedra", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "layers": [{"type": t, "mixer": mixers[t], "mlp": {"kind": "dense", "ff": s["ff"]}} for t in BAGEDRA_LAYERS]}


def bobavik_like(s: dict) -> dict:
    """Bobavik with Bagedra's width, heads, layer order and feed-forward"""
    mlp = {"kind": "moe", "expert": {"ff": s["ff"]}, "router": {"experts": 1, "top": 1}, "shared": None}
    soft = {"heads": s["heads"], "kv_heads": s["heads"] // 4, "dim": s["dim"], "vdim": s["dim"], "scale": s["dim"] ** -0.5, "v_mix": False,
            "rot": {"dims": s["dim"], "base": 500000.0}}
    lin = {"heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "decay": [0.9 + 0.099 * i / s["heads"] for i in range(s["heads"])]}
    return {"architecture": "Bobavik", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "logit_scale": 1.0,
            "layers": [{"type": "attention" if t == "latent_attention" else "lightning", "mixer": soft if t == "latent_attention" else lin,
                        "mlp": mlp} for t in BAGEDRA_LAYERS]}


def design_config(s: dict) -> dict:
    mlp = {"kind": "moe", "expert": {"ff": s["ff"]}, "router": {"experts": s["experts"], "top": s["top"]}, "shared": {"ff": s["shared"]}}
    soft = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": s["dim"] ** -0.5, "v_mix": True,
            "mask": {"size": s["window"]}, "rot": {"dims": s["dim"], "base": 500000.0}}
    lin = {"heads": s["heads"], "dim": s["dim"], "vdim": s["dim"], "decay": [0.9 + 0.099 * i / s["heads"] for i in range(s["heads"])]}
    return {"architecture": "Bobavik", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "logit_scale": 1.0,
            "layers": [{"type": t, "mixer": soft if t == "attention" else lin, "mlp": mlp} for t in LAYERS]}


class RandomState(dict):
    """Weights drawn on the device when they are asked for: matrices of unit gain, norms near one."""

    def __init__(self, device, seed=0):
        self.device, self.gen = device, torch.Generator(device=device)
        self.gen.manual_seed(seed)

    def __contains__(self, name):
        return True

    def __missing__(self, name):
        return _Lazy(self, name)


class _Lazy:
    """A tensor of whatever shape the loader expects."""

    def __init__(self, state, name):
        self.state, self.name = state, name

    def draw(self, shape):
        s = self.state
        t = torch.randn(shape, generator=s.gen, device=s.device, dtype=torch.bfloat16)
        if len(shape) == 2:
            return t.mul_(shape[1] ** -0.5)
        return (0.02 * t) if self.name.endswith(".b") else (1.0 + 0.02 * t) if len(shape) else torch.tensor(0.5)


def random_model(config: dict, device, rank=None, seed=0):
    from ..backend.lm import lm_ops
    from ..models import layers
    cls = model_class(config)

    class Drawn(layers.Weights):
        def rows(self, name):
            return rank

        def under(self, prefix):
            return Drawn(self.state, self.device, self.dtype, self.prefix + prefix, self.used)

        def raw(self, name, *shape):
            return self.state[self.prefix + name].draw(shape)

    return cls(sys.modules[cls.__module__].parse_config(config), Drawn(RandomState(device, seed), device, torch.bfloat16), lm_ops(torch.bfloat16))


def _timed(fn, reps):
    fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(reps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / reps


def measure_design(config: dict, device, rank=None, batches=(16, 64), context=1024, steps=32, prompt=16384):
    s, model = config, random_model(config, device, rank)
    gen = torch.Generator().manual_seed(1)
    draw = lambda n: torch.randint(0, s["vocab"], (n,), generator=gen).tolist()      # noqa: E731
    out = {}
    engine = Engine(model, max_tokens=max(max(batches) * (context + 128), prompt + 64), max_seqs=max(batches))
    one = draw(prompt)

    def whole(parts):
        seqs = [engine.open() for _ in range(parts)]
        n = prompt // parts
        engine.run([SequenceInput(q, one[i * n:(i + 1) * n], [n - 1]) for i, q in enumerate(seqs)])
        for q in seqs:
            engine.close(q)

    for parts in (1, 16):
        t = _timed(lambda: whole(parts), 3)
        out["prefill_%dx%d" % (parts, prompt // parts)] = {"ms": round(t * 1e3, 3), "tokens_per_s": round(prompt / t, 1)}
    for B in batches:
        seqs = [engine.open() for _ in range(B)]
        for i in range(0, B, 16):
            engine.run([SequenceInput(q, one[:context], []) for q in seqs[i:i + 16]])
        # the engine's own loop: schedule-free single tokens, greedy choice on the device, token ids through the host
        tokens = draw(B)

        def step():
            nonlocal tokens
            z = engine.run([SequenceInput(q, [t], [0]) for q, t in zip(seqs, tokens)])
            tokens = model.greedy(z).tolist()

        t = _timed(step, steps)
        key = next(k for k in engine._graphs if k[0] >= B)
        graph = engine._graphs[key][1]
        g = _timed(graph.run, steps)            # the captured step alone, replayed without new metadata
        out["decode_bs%d" % B] = {"ms_per_step": round(t * 1e3, 4), "graph_ms": round(g * 1e3, 4), "tokens_per_s": round(B / t, 1)}
        for q in seqs:
            engine.close(q)
    return out


def measure_llama(size: str, device, batches=(16, 64), context=1024, steps=32, prompt=16384):
    s = SIZES[size]
    cfg = LlamaConfig(hidden=s["width"], inter=s["top"] * s["ff"] + s["shared"], heads=s["heads"], kv_heads=s["kv_heads"],
                      head_dim=s["dim"], layers=len(LAYERS), vocab=s["vocab"])
    out = {}
    for parts, ctx in ((1, prompt), (16, prompt // 16)):
        r = DecodeRunner(cfg, parts, ctx, 8, device, seed=2)
        t = _timed(lambda: r.prefill(ctx), 3)
        out["prefill_%dx%d" % (parts, ctx)] = {"ms": round(t * 1e3, 3), "tokens_per_s": round(prompt / t, 1)}
        del r
    for B in batches:
        r = DecodeRunner(cfg, B, context, 4 * steps + 16, device, seed=2)
        t = _timed(r.step, steps)
        out["decode_bs%d" % B] = {"ms_per_step": round(t * 1e3, 4), "tokens_per_s": round(B / t, 1)}
        del r
        gc.collect()
        torch.cuda.empty_cache()
    return out


def run(device, sizes=tuple(SIZES), llama=True):
    res = {}
    for size in sizes:
        res[size] = {"sizes": SIZES[size], "layers": LAYERS, "bobavik_bf16": measure_design(design_config(SIZES[size]), device)}
        gc.collect()
        torch.cuda.empty_cache()
        if llama:
            res[size]["llama_w4a8kv4"] = measure_llama(size, device)
            gc.collect()
            torch.cuda.empty_cache()
    return res


def run_bagedra(device, sizes=tuple(BAGEDRA_SIZES), beside=True):
    res = {}
    for size in sizes:
        s = BAGEDRA_SIZES[size]
        res[size] = {"sizes": s, "layers": BAGEDRA_LAYERS}
        for name, config in (("bagedra_bf16", bagedra_config(s)), ("bobavik_bf16", bobavik_like(s)))[:2 if beside else 1]:
            res[size][name] = measure_design(config, device, s["rank"])
            gc.collect()
            torch.cuda.empty_cache()
    return res
