"""Plain float64 restatement of the Bagedra decoder (numpy, one function per mechanism, no caching, no batching, whole sequences
only): latent attention, gated linear attention, the gated delta rule, dense gated feed-forward.  Shares no code with
omniserve_amd.

Every function takes the sequence as [tokens, features] arrays and a dictionary of weights; linear weights are [out, in].
"""
import numpy as np

from .hybrid import f64, linear, rms_norm, rope_frequencies, sigmoid, silu, under


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rotate_halves(x, positions, freqs):
    """x [tokens, heads, dim]: dimension i paired with i + len(freqs), turned by position * freqs[i]."""
    n = len(freqs)
    a = f64(positions)[:, None] * freqs[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * n:]], axis=-1)


# ---- latent attention ----------------------------------------------------------------------------------------------
def latent(h, W, m, eps, positions=None):
    """-> (latent [T, kv_rank], rotated key part [T, rot_dim]) that all heads share"""
    pos = np.arange(h.shape[0]) if positions is None else positions
    y = linear(h, W["dkv"])
    c = rms_norm(y[:, :m["kv_rank"]], W["dkv.norm"], eps)
    fr = rope_frequencies(m["rot"]["dims"], m["rot"]["base"])
    return c, rotate_halves(y[:, None, m["kv_rank"]:], pos, fr)[:, 0]


def latent_attention(q, c, kr, uk, uv, scale, heads, vdim):
    """q [T, H, dim + rot_dim] (turned), c [T, R], kr [T, rot_dim] -> [T, H, vdim]; position i attends to every j <= i"""
    T, dim = q.shape[0], q.shape[2] - kr.shape[1]
    k = linear(c, uk).reshape(T, heads, dim)
    v = linear(c, uv).reshape(T, heads, vdim)
    seen = np.tril(np.ones((T, T), bool))
    out = np.zeros((T, heads, vdim))
    for h in range(heads):
        s = (q[:, h, :dim] @ k[:, h].T + q[:, h, dim:] @ kr.T) * scale
        s = np.where(seen, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h]
    return out


def latent_attention_mixer(h, W, m, shared, eps, positions=None):
    """-> (output, (latent, rotated key part)); shared: those of another layer, or None when the layer has its own"""
    T, H = h.shape[0], m["heads"]
    pos = np.arange(T) if positions is None else positions
    q = linear(h, W["q"]).reshape(T, H, m["dim"] + m["rot_dim"])
    fr = rope_frequencies(m["rot"]["dims"], m["rot"]["base"])
    q = np.concatenate([q[..., :m["dim"]], rotate_halves(q[..., m["dim"]:], pos, fr)], axis=-1)
    c, kr = latent(h, W, m, eps, pos) if shared is None else shared
    o = latent_attention(q, c, kr, W["uk"], W["uv"], m["scale"], H, m["vdim"]).reshape(T, -1)
    return linear(o * sigmoid(linear(h, W["g"])), W["o"]), (c, kr)


# ---- recurrences -----------------------------------------------------------------------------------------------------
def gated_linear_attention(q, k, v, log_alpha, state=None):
    """q, k, log_alpha [T, H, D], v [T, H, E]: S <- diag(alpha) S + k v^T, o = S^T q, token by token -> (o, S)"""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2])) if state is None else f64(state).copy()
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = np.exp(log_alpha[t])[:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.matmul(q[t][:, None, :], S)[:, 0]
    return out, S


def gla_log_decay(h, W, m):
    z = linear(linear(h, W["a1"]), W["a2"]) + f64(W["a2.b"])
    return (-softplus(-z) / m["tau"]).reshape(h.shape[0], m["heads"], m["dim"])


def gla_mixer(h, W, m, eps):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = linear(h, W["q"]).reshape(T, H, D) * D ** -0.5
    k = linear(h, W["k"]).reshape(T, H, D)
    v = linear(h, W["v"]).reshape(T, H, E)
    o, _ = gated_linear_attention(q, k, v, gla_log_decay(h, W, m))
    o = rms_norm(o, W["norm"], eps).reshape(T, H * E)
    return linear(o * silu(linear(h, W["g"])), W["o"])


def short_convolution(x, w):
    """x [T, C], w [C, taps]: the last column of w meets the current token, zeros before the start"""
    T, taps = x.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(padded[i:i + T] * f64(w)[:, i] for i in range(taps))


def unit(x):
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)


def gated_delta_rule(q, k, v, log_g, beta, state=None):
    """q, k [T, H, D], v [T, H, E], log_g, beta [T, H] -> (o [T, H, E], S)"""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2])) if state is None else f64(state).copy()
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = np.exp(log_g[t])[:, None, None] * S
        u = beta[t][:, None] * (v[t] - np.matmul(k[t][:, None, :], S)[:, 0])
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.matmul(q[t][:, None, :], S)[:, 0]
    return out, S


def delta_gates(h, W):
    """-> (logarithm of the decay, step size), [T, heads] each"""
    log_g = -np.exp(f64(W["A_log"])) * softplus(linear(h, W["a"]) + f64(W["dt_bias"]))
    return log_g, sigmoid(linear(h, W["b"]))


def delta_mixer(h, W, m, eps):
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: silu(short_convolution(linear(h, W[n]), W[n + ".conv"]))      # noqa: E731
    q = unit(conv("q").reshape(T, G, D)) * D ** -0.5
    k = unit(conv("k").reshape(T, G, D))
    v = conv("v").reshape(T, H, E)
    q, k = np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1)
    o, _ = gated_delta_rule(q, k, v, *delta_gates(h, W))
    o = rms_norm(o, W["norm"], eps).reshape(T, H * E)
    return linear(o * silu(linear(h, W["g"])), W["o"])


# ---- feed-forward, decoder -------------------------------------------------------------------------------------------
def dense(h, W):
    a = gelu_tanh(linear(h, W["gate"]) + f64(W["gate.b"])) * (linear(h, W["up"]) + f64(W["up.b"]))
    return linear(a, W["down"]) + f64(W["down.b"])


def decoder(cfg, weights, tokens):
    """-> (logits [T, vocab], residual after every layer [layers, T, width])."""
    eps = cfg["norm"]["eps"]
    x = f64(weights["embed"])[np.asarray(tokens)] * cfg["embedding"]["scale"]
    shared, after = {}, []
    for i, layer in enumerate(cfg["layers"]):
        L = "l%d." % i
        W, m = under(weights, L + "mix."), layer["mixer"]
        if layer["type"] == "latent_attention":
            y, shared[i] = latent_attention_mixer(x, W, m, shared[m["kv_from"]] if m.get("kv_from") is not None else None, eps)
        else:
            y = (gla_mixer if layer["type"] == "gla" else delta_mixer)(x, W, m, eps)
        x = x + rms_norm(y, weights[L + "norm1"], eps)
        if layer.get("mlp"):
            x = x + rms_norm(dense(x, under(weights, L + "mlp.")), weights[L + "norm2"], eps)
        after.append(x)
    return linear(rms_norm(x, weights["final.norm"], eps), weights["head"]), np.stack(after)
