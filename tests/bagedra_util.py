"""Small random models of the Bagedra decoder for the tests: configurations and weights."""
import torch


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def latent(heads=5, dim=24, rot_dim=12, vdim=40, kv_rank=56, base=20000.0, scale=None, kv_from=None, mlp=True, ff=72):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": {"dims": rot_dim, "base": base},
         "scale": scale or 1.6 / (dim + rot_dim) ** 0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": dense(ff) if mlp else None}


def gla(heads=3, dim=40, vdim=72, tau=6.0, rank=10, mlp=True, ff=72):
    """(rank: of the decays' projection; the checkpoint's shapes carry it)"""
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": dense(ff) if mlp else None, "rank": rank}


def delta(heads=4, kv_heads=2, dim=24, vdim=40, conv=3, mlp=True, ff=72):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": dense(ff) if mlp else None}


def config(layers, width=104, vocab=211, eps=1e-4, embed_scale=3.0):
    return {"architecture": "Bagedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
            "layers": layers}


def tensors(cfg):
    """name -> (shape, spread of its random values, their mean)"""
    W, out = cfg["width"], {}

    def mat(name, n, k, gain=1.0):
        out[name] = ((n, k), gain / k ** 0.5, 0.0)

    # (inputs of a sublayer are the residual itself: the embeddings are of unit size after their scale)
    out["embed"] = ((cfg["vocab"], W), 1.0 / cfg["embedding"]["scale"], 0.0)
    mat("head", cfg["vocab"], W)
    out["final.norm"] = ((W,), 0.3, 1.0)
    for i, l in enumerate(cfg["layers"]):
        p, m, x = "l%d." % i, l["mixer"], "l%d.mix." % i
        out[p + "norm1"] = ((W,), 0.2, 0.7)
        if l["mlp"]:
            ff = l["mlp"]["ff"]
            out[p + "norm2"] = ((W,), 0.2, 0.7)
            for n, a, b in (("gate", ff, W), ("up", ff, W), ("down", W, ff)):
                mat(p + "mlp." + n, a, b)
                out[p + "mlp." + n + ".b"] = ((a,), 0.4, 0.0)
        H, D, E = m["heads"], m["dim"], m["vdim"]
        mat(x + "g", H * E, W), mat(x + "o", W, H * E)
        if l["type"] == "latent_attention":
            R, rot = m["kv_rank"], m["rot_dim"]
            mat(x + "q", H * (D + rot), W, 1.5), mat(x + "uk", H * D, R, 1.5), mat(x + "uv", H * E, R)
            if m.get("kv_from") is None:
                mat(x + "dkv", R + rot, W)
                out[x + "dkv.norm"] = ((R,), 0.3, 1.0)
        elif l["type"] == "gla":
            mat(x + "q", H * D, W), mat(x + "k", H * D, W), mat(x + "v", H * E, W)
            mat(x + "a1", l["rank"], W), mat(x + "a2", H * D, l["rank"], 1.5)
            out[x + "a2.b"], out[x + "norm"] = ((H * D,), 1.0, 1.0), ((E,), 0.3, 1.0)
        else:
            G, C = m["kv_heads"], m["conv"]
            for n, c in (("q", G * D), ("k", G * D), ("v", H * E)):
                mat(x + n, c, W)
                out[x + n + ".conv"] = ((c, C), 0.7, 0.3)
            mat(x + "a", H, W), mat(x + "b", H, W)
            out[x + "A_log"], out[x + "dt_bias"], out[x + "norm"] = ((H,), 0.8, 0.0), ((H,), 1.0, -2.5), ((E,), 0.3, 1.0)
    return out


def random_state(cfg, seed=0):
    """bf16 weights, so that both number formats and the oracle work on the same values"""
    g = torch.Generator().manual_seed(seed)
    return {n: (mean + spread * torch.randn(shape, generator=g)).bfloat16() for n, (shape, spread, mean) in tensors(cfg).items()}


MODELS = {
    "mixed": config([gla(), delta(), latent(), gla(heads=2, dim=72, vdim=24, tau=1.0, rank=3, mlp=False), latent(kv_from=2, heads=18, vdim=72),
                     delta(heads=3, kv_heads=1, conv=4), latent(kv_rank=72, heads=1, dim=40, rot_dim=32)]),
    "latent only": config([latent(mlp=False), latent(kv_from=0, dim=70, mlp=False)], width=72, vocab=90, embed_scale=1.0),
    "shared by two": config([latent(kv_rank=130, rot_dim=8), gla(tau=1.0), latent(kv_rank=130, rot_dim=8, kv_from=0, heads=2),
                             latent(kv_rank=130, rot_dim=8, kv_from=0, heads=3, vdim=16)], width=136, vocab=65, eps=1e-6),
    "recurrent only": config([delta(conv=1, heads=2, kv_heads=2), gla(heads=1), delta(conv=6, dim=72, vdim=136, ff=200)], width=64, vocab=130),
}
