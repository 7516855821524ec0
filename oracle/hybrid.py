"""Plain float64 restatement of the hybrid decoder layers the engine serves (numpy, one function per mechanism, no caching,
no batching, whole sequences only).  Shares no code with omniserve_amd.

Every function takes the sequence as [tokens, features] arrays and a dictionary of weights; linear weights are [out, in].
"""
import math

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def linear(x, w):
    return x @ f64(w).T


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def layer_norm(x, w, b, eps):
    m = x.mean(axis=-1, keepdims=True)
    d = x - m
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * f64(w) + f64(b)


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * f64(w)


def rope_frequencies(dims, base, scaling=None):
    """Rotation per position of each pair.  `scaling`: the three-band rule -- short wavelengths kept, long ones stretched by
    `factor`, a linear blend in between -- with band edges original / high and original / low."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            n = scaling["original"] / wave
            if wave < scaling["original"] / scaling["high"]:
                pass
            elif wave > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            else:
                s = (n - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate_pairs(x, positions, freqs):
    """x [tokens, heads, dim]: pair (2i, 2i + 1) of every head turned by position * freqs[i]; dims past the pairs unchanged."""
    y = x.copy()
    a = f64(positions)[:, None] * freqs[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    n = 2 * len(freqs)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2] = u * c - v * s
    y[..., 1:n:2] = v * c + u * s
    return y


def windowed_attention(q, k, v, scale, window):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; position i attends to (i - window, i]."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    i = np.arange(T)
    seen = (i[:, None] >= i[None, :]) & (i[:, None] - i[None, :] < window)
    for h in range(H):
        s = (q[:, h] @ k[:, h // group].T) * scale
        s = np.where(seen, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h // group]
    return out


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attention_mixer(h, W, m, v_first, positions=None):
    """-> (output, this layer's unmixed values).  v_first: the values of the first value-mixing layer, None in that layer or
    when the layer does not mix."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = np.arange(T) if positions is None else positions
    q = linear(h, W["q"]).reshape(T, H, D)
    k = linear(h, W["k"]).reshape(T, G, D)
    v = linear(h, W["v"]).reshape(T, G, E)
    raw = v
    if v_first is not None:
        v = mix_values(v, v_first, float(W["vmix"]))
    if m.get("rot"):
        fr = rope_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
        q, k = rotate_pairs(q, pos, fr), rotate_pairs(k, pos, fr)
    o = windowed_attention(q, k, v, m["scale"], m["mask"]["size"] if m.get("mask") else T + 1).reshape(T, H * E)
    return linear(o * sigmoid(linear(h, W["g"])), W["o"]), raw


def decayed_linear_attention(q, k, v, decay, state=None):
    """q, k [T, H, D], v [T, H, E] -> ([T, H, E], final state [H, D, E]); S <- decay S + k v^T, o = S^T q, token by token."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2])) if state is None else f64(state).copy()
    lam = f64(decay)[:, None, None]
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = lam * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hd,hde->he", q[t], S)
    return out, S


def lightning_mixer(h, W, m, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = silu(linear(h, W["q"])).reshape(T, H, D)
    k = silu(linear(h, W["k"])).reshape(T, H, D)
    v = silu(linear(h, W["v"])).reshape(T, H, E)
    o, _ = decayed_linear_attention(q, k, v, m["decay"])
    o = rms_norm(o.reshape(T, H * E), W["norm"], eps)
    return linear(o * sigmoid(linear(h, W["g"])), W["o"])


def glu(h, gate, up, down):
    return linear(silu(linear(h, gate)) * linear(h, up), down)


def route(h, router, bias, top):
    """-> (expert ids [T, top], weights [T, top]): the `top` largest logits, softmax over those alone."""
    z = linear(h, router) + f64(bias)
    ids = np.argsort(-z, axis=1, kind="stable")[:, :top]
    zc = np.take_along_axis(z, ids, axis=1)
    e = np.exp(zc - zc.max(axis=1, keepdims=True))
    return ids, e / e.sum(axis=1, keepdims=True)


def mixture(h, W, m):
    ids, wt = route(h, W["router"], W["router.b"], m["router"]["top"])
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(ids[t], wt[t]):
            y[t] += w * glu(h[t:t + 1], W["e%d.gate" % e], W["e%d.up" % e], W["e%d.down" % e])[0]
    if m.get("shared"):
        y += glu(h, W["shared.gate"], W["shared.up"], W["shared.down"])
    return y


def under(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def decoder(cfg, weights, tokens):
    """-> (logits [T, vocab], residual after every layer [layers, T, width])."""
    eps = cfg["norm"]["eps"]
    x = f64(weights["embed"])[np.asarray(tokens)]
    v_first, after = None, []
    for i, layer in enumerate(cfg["layers"]):
        L = "l%d." % i

        def norm(name, z):
            return layer_norm(z, weights[L + name], weights[L + name + ".b"], eps)

        W, m = under(weights, L + "mix."), layer["mixer"]
        h = norm("norm1", x)
        if layer["type"] == "attention":
            y, raw = attention_mixer(h, W, m, v_first if m.get("v_mix") else None)
            if m.get("v_mix") and v_first is None:
                v_first = raw
        else:
            y = lightning_mixer(h, W, m, eps)
        x = x + norm("norm1b", y)
        if layer.get("mlp"):
            x = x + norm("norm2b", mixture(norm("norm2", x), under(weights, L + "mlp."), layer["mlp"]))
        after.append(x)
    h = layer_norm(x, weights["final.norm"], weights["final.norm.b"], eps)
    return linear(h, weights["head"]) * cfg["logit_scale"], np.stack(after)
