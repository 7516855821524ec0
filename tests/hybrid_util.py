"""Small random models of the hybrid decoder for the tests: configurations, weights, and running them in pieces."""
import numpy as np
import torch


def attention(heads=4, kv_heads=2, dim=48, vdim=40, window=37, rot=32, base=10000.0, scale=None, v_mix=True, scaling=True, mlp="moe", **moe_kw):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or 1.7 / dim ** 0.5, "v_mix": v_mix,
         "mask": {"size": window}}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if scaling:
            m["rot"]["scaling"] = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 200}
    return {"type": "attention", "mixer": m, "mlp": moe(**moe_kw) if mlp else None}


def lightning(heads=3, dim=40, vdim=72, decay=None, mlp="moe", **moe_kw):
    decay = decay or [0.55, 0.93, 0.9985, 1.0, 0.99, 0.7][:heads]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay},
            "mlp": moe(**moe_kw) if mlp else None}


def moe(experts=6, top=2, ff=48, shared=80):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}


def config(layers, width=160, vocab=301, eps=1e-5, logit_scale=0.4):
    return {"architecture": "Bobavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}


def tensors(cfg):
    """name -> (shape, spread of its random values, their mean)"""
    W, out = cfg["width"], {}

    def mat(name, n, k, gain=1.0):
        out[name] = ((n, k), gain / k ** 0.5, 0.0)

    def norm(name):
        out[name], out[name + ".b"] = ((W,), 0.3, 1.0), ((W,), 0.2, 0.0)

    out["embed"] = ((cfg["vocab"], W), 1.0, 0.0)
    mat("head", cfg["vocab"], W)
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] else ()):
            norm(p + n)
        H, D, E = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "attention":
            G = m["kv_heads"]
            mat(p + "mix.q", H * D, W, 1.5), mat(p + "mix.k", G * D, W, 1.5), mat(p + "mix.v", G * E, W)
            if m["v_mix"]:
                out[p + "mix.vmix"] = ((), 0.1, 0.45)
        else:
            mat(p + "mix.q", H * D, W, 1.5), mat(p + "mix.k", H * D, W, 1.5), mat(p + "mix.v", H * E, W, 1.5)
            out[p + "mix.norm"] = ((H * E,), 0.3, 1.0)
        mat(p + "mix.g", H * E, W, 2.0), mat(p + "mix.o", W, H * E)
        if l["mlp"]:
            f, q = l["mlp"], p + "mlp."
            mat(q + "router", f["router"]["experts"], W, 3.0)
            out[q + "router.b"] = ((f["router"]["experts"],), 0.5, 0.0)
            parts = [("e%d." % e, f["expert"]["ff"]) for e in range(f["router"]["experts"])]
            if f["shared"]:
                parts.append(("shared.", f["shared"]["ff"]))
            for n, ff in parts:
                mat(q + n + "gate", ff, W, 2.0), mat(q + n + "up", ff, W), mat(q + n + "down", W, ff)
    return out


def random_state(cfg, seed=0):
    """bf16 weights, so that both number formats and the oracle work on the same values"""
    g = torch.Generator().manual_seed(seed)
    return {n: (mean + spread * torch.randn(shape, generator=g)).bfloat16() for n, (shape, spread, mean) in tensors(cfg).items()}


def to_numpy(state):
    return {k: v.double().numpy() for k, v in state.items()}


def random_tokens(cfg, n, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def cuts(n, sizes):
    """portions of the sizes in turn until n tokens are cut"""
    out, i = [], 0
    while sum(out) < n:
        out.append(min(sizes[i % len(sizes)], n - sum(out)))
        i += 1
    return out


def run_alone(engine, tokens, sizes):
    """logits at every position, the sequence cut into portions of `sizes`"""
    from omniserve_amd.engine import SequenceInput
    seq, at, out = engine.open(), 0, []
    for n in cuts(len(tokens), sizes):
        out.append(engine.run([SequenceInput(seq, tokens[at:at + n], list(range(n)))]).cpu())
        at += n
    engine.close(seq)
    return torch.cat(out).numpy()


def errors(got, want):
    """per position: rms of the difference over the rms of all expected values"""
    d = np.asarray(got, np.float64) - want
    return np.sqrt((d * d).mean(axis=-1) / (want * want).mean())
