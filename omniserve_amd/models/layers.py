"""Building blocks of the decoder models the engine serves: specifications (sizes and constants) and the layers that run them on
the kernels of backend/lm.py.

Inner sizes are padded with zeros when the weights are loaded -- the model width and the feed-forward to multiples of 64, every
head to 64, 128 or 256 -- so that the kernels' k loops carry no bounds.  A padded q / k dimension adds zero to every score, a
padded value column meets a zero column of the output projection; statistics of norms use the real sizes."""
from __future__ import annotations

import dataclasses
import math
from typing import List, Optional, Tuple

import torch

from ..backend.lm import ATTN_ROWS, PAGE, LmOps
from ..rope import inverse_frequencies
from .base import EngineModel

NO_WINDOW = 1 << 30


# ---------------------------------------------------------------------------------------------------------------
# specifications
# ---------------------------------------------------------------------------------------------------------------
@dataclasses.dataclass(frozen=True)
class RotarySpec:
    dims: int                         # leading dimensions of a head that turn, in neighbouring pairs
    base: float
    scaling: Optional[dict] = None    # factor, low, high, original: see rope.inverse_frequencies


@dataclasses.dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None      # newest positions a token attends to, its own included; None: all
    rotary: Optional[RotarySpec] = None
    value_mix: bool = False           # blend the values with those of the model's first value-mixing layer
    gate: bool = True                 # sigmoid(W_g h) on the heads' output

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if not self.scale > 0:
            raise ValueError("the score scale must be positive")
        if self.window is not None and self.window < 1:
            raise ValueError("a window holds at least the token itself")
        if self.rotary is not None and (self.rotary.dims % 2 or self.rotary.dims > self.dim):
            raise ValueError("rotary dims must be even and at most the head size")


@dataclasses.dataclass(frozen=True)
class LinearAttentionSpec:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]          # per head
    activation: Optional[str] = "silu"

    def __post_init__(self):
        if len(self.decay) != self.heads:
            raise ValueError("one decay per head")
        if not all(0.0 <= d <= 1.0 for d in self.decay):
            raise ValueError("decays lie in [0, 1]")


@dataclasses.dataclass(frozen=True)
class MoeSpec:
    experts: int
    top: int
    ff: int
    shared_ff: Optional[int] = None

    def __post_init__(self):
        if not 1 <= self.top <= self.experts:
            raise ValueError("a token uses between 1 and all experts")


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: object                     # AttentionSpec or LinearAttentionSpec
    moe: Optional[MoeSpec]


@dataclasses.dataclass(frozen=True)
class DecoderSpec:
    vocab: int
    width: int
    layers: Tuple[LayerSpec, ...]
    eps: float
    norm: str = "layer"               # "layer" (weight and bias) or "rms" (weight)
    logit_scale: float = 1.0


# ---------------------------------------------------------------------------------------------------------------
# padding
# ---------------------------------------------------------------------------------------------------------------
def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def pad_head(n: int) -> int:
    for p in (64, 128, 256):
        if n <= p:
            return p
    raise ValueError("head size %d is larger than the kernels' 256" % n)


def padded(t: torch.Tensor, *sizes) -> torch.Tensor:
    """t in the corner of a zero tensor of these sizes."""
    if tuple(t.shape) == tuple(sizes):
        return t.contiguous()
    out = t.new_zeros(sizes)
    out[tuple(slice(0, s) for s in t.shape)] = t
    return out


def pad_out_heads(w, heads, dim, width):
    """[heads * dim, in] -> [heads * pad_head(dim), width]"""
    return padded(w.reshape(heads, dim, w.shape[1]), heads, pad_head(dim), width).reshape(heads * pad_head(dim), width)


def pad_in_heads(w, heads, dim, rows):
    """[out, heads * dim] -> [rows, heads * pad_head(dim)]"""
    return padded(w.reshape(w.shape[0], heads, dim), rows, heads, pad_head(dim)).reshape(rows, heads * pad_head(dim))


def pair_rows(gate, up, ff, width):
    """gate, up [n, in] -> [2 ff, width], blocks of 16 rows of each in turn (the gated epilogue's order)."""
    g, u = padded(gate, ff, width).reshape(ff // 16, 16, width), padded(up, ff, width).reshape(ff // 16, 16, width)
    return torch.stack((g, u), dim=1).reshape(2 * ff, width)


class Weights:
    """A checkpoint's tensors under one prefix; every tensor is looked up by name, checked for its shape and counted, so that
    leftovers can be reported."""

    def __init__(self, state, device, dtype, prefix="", used=None):
        self.state, self.device, self.dtype, self.prefix = state, device, dtype, prefix
        self.used = set() if used is None else used

    def under(self, prefix):
        return Weights(self.state, self.device, self.dtype, self.prefix + prefix, self.used)

    def raw(self, name, *shape):
        full = self.prefix + name
        if full not in self.state:
            raise RuntimeError("the checkpoint lacks tensor %s" % full)
        t = self.state[full]
        if tuple(t.shape) != shape:
            raise RuntimeError("checkpoint tensor %s has shape %s, the model expects %s" % (full, tuple(t.shape), shape))
        self.used.add(full)
        return t

    def matrix(self, name, *shape):
        return self.raw(name, *shape).to(device=self.device, dtype=self.dtype)

    def vector(self, name, n, size=None):
        """f32, padded with zeros to `size`"""
        return padded(self.raw(name, n).to(device=self.device, dtype=torch.float32), size or n)

    def scalar(self, name):
        return float(self.raw(name))

    def leftovers(self, optional=()):
        return sorted(k for k in self.state if k not in self.used and not any(k.endswith(o) for o in optional))


# ---------------------------------------------------------------------------------------------------------------
# layers
# ---------------------------------------------------------------------------------------------------------------
class Norm:
    def __init__(self, w: Weights, name: str, width: int, size: int, kind: str):
        self.pair = (w.vector(name, width, size), w.vector(name + ".b", width, size) if kind == "layer" else None)


class Attention:
    """Grouped-query softmax attention over the paged cache: sliding window, rotary positions, value mixing, output gate."""

    def __init__(self, s: AttentionSpec, w: Weights, ops: LmOps, width: int, mixes: bool):
        self.s, self.ops = s, ops
        H, G, W = s.heads, s.kv_heads, pad64(width)
        self.dk, self.dv = pad_head(s.dim), pad_head(s.vdim)
        parts = [pad_out_heads(w.matrix("q", H * s.dim, width), H, s.dim, W),
                 pad_out_heads(w.matrix("k", G * s.dim, width), G, s.dim, W),
                 pad_out_heads(w.matrix("v", G * s.vdim, width), G, s.vdim, W)]
        self.nq, self.nv, self.v0 = H * self.dk, G * self.dv, (H + G) * self.dk
        self.g0 = self.v0 + self.nv
        if s.gate:
            parts.append(pad_out_heads(w.matrix("g", H * s.vdim, width), H, s.vdim, W))
        self.w_in = torch.cat(parts)
        self.w_out = pad_in_heads(w.matrix("o", width, H * s.vdim), H, s.vdim, W)
        self.lam = w.scalar("vmix") if mixes else 0.0     # mixes: value_mix, and not the first layer that has it
        self.mixes = mixes
        freq = inverse_frequencies(s.rotary.dims, s.rotary.base, s.rotary.scaling) if s.rotary else []
        self.freq = torch.tensor(freq, dtype=torch.float64).to(device=w.device, dtype=torch.float32)
        self.window = s.window or NO_WINDOW

    def cache_shape(self):
        return self.s.kv_heads, self.dk, self.dv

    def __call__(self, h, b, kv, v_first):
        """-> (output, this layer's unmixed values)"""
        s, ops = self.s, self.ops
        x = ops.matmul(h, self.w_in)
        o = torch.empty((h.shape[0], s.heads * self.dv), dtype=h.dtype, device=h.device)
        v = x[:, self.v0:self.v0 + self.nv]
        gate = x[:, self.g0:] if s.gate else None
        first = v_first if self.mixes else None
        heads = (s.heads, s.kv_heads, self.dk, self.dv)
        n = b.n_prompt
        cut = lambda t, lo, hi: None if t is None else t[lo:hi]      # noqa: E731
        if n:
            ops.rope_append(x[:n], cut(first, 0, n), self.lam, self.freq, b.pos, b.kv_slot, kv[0], kv[1], *heads)
            ops.attn_prefill(x[:n], kv[0], kv[1], b.block_table, b.entry, b.attn_tiles, cut(gate, 0, n), o[:n], s.scale, self.window, *heads)
        if b.n_decode:
            nsplit = self.splits(b)
            part = None
            if nsplit > 1:
                part = torch.empty((b.n_decode * s.heads * nsplit * (self.dv + 2),), dtype=torch.float32, device=h.device)
            ops.attn_decode(x[n:], cut(first, n, None), self.lam, self.freq, b.pos[n:], b.kv_slot[n:], kv[0], kv[1],
                            b.block_table[b.n_entries:], cut(gate, n, None), o[n:], part, nsplit, s.scale, self.window, *heads)
        return ops.matmul(o, self.w_out), v

    def splits(self, b) -> int:
        """Parts of the visible keys per (sequence, kv head): enough workgroups for the 256 CUs, at least 128 keys each."""
        keys = min(self.window, b.max_context)
        groups = b.n_decode * self.s.kv_heads * ((self.s.heads // self.s.kv_heads + 15) // 16)
        return max(1, min(512 // max(groups, 1), keys // 128, 64))


class LinearAttention:
    """Decayed linear attention with an RMS norm over the concatenated heads and an output gate."""

    def __init__(self, s: LinearAttentionSpec, w: Weights, ops: LmOps, width: int, eps: float):
        self.s, self.ops, self.eps = s, ops, eps
        H, W = s.heads, pad64(width)
        self.dk, self.dv = pad_head(s.dim), pad_head(s.vdim)
        self.w_in = torch.cat([pad_out_heads(w.matrix("q", H * s.dim, width), H, s.dim, W),
                               pad_out_heads(w.matrix("k", H * s.dim, width), H, s.dim, W),
                               pad_out_heads(w.matrix("v", H * s.vdim, width), H, s.vdim, W),
                               pad_out_heads(w.matrix("g", H * s.vdim, width), H, s.vdim, W)])
        self.g0 = 2 * H * self.dk + H * self.dv
        self.w_out = pad_in_heads(w.matrix("o", width, H * s.vdim), H, s.vdim, W)
        self.norm = pad_in_heads(w.vector("norm", H * s.vdim)[None], H, s.vdim, 1)[0].contiguous()
        self.log2_decay = torch.tensor([math.log2(d) if d > 0 else -1e30 for d in s.decay], dtype=torch.float64).to(device=w.device, dtype=torch.float32)

    def state_shape(self):
        return self.s.heads, self.dk, self.dv

    def __call__(self, h, b, state):
        s, ops, n = self.s, self.ops, b.n_prompt
        x = ops.matmul(h, self.w_in)
        o = torch.empty((h.shape[0], s.heads * self.dv), dtype=h.dtype, device=h.device)
        size = (s.heads, self.dk, self.dv)
        if n:
            seg_state = None
            if b.multi_segment:
                seg_state = torch.empty((b.segments.shape[0],) + size, dtype=torch.float32, device=h.device)
            ops.linear_prefill(x[:n], o[:n], state, seg_state, b.segments, b.segment_len, b.multi_segment, self.log2_decay, *size,
                               s.activation)
        if b.n_decode:
            ops.linear_decode(x[n:], o[n:], state, b.state_slot, b.pos[n:], self.log2_decay, *size, s.activation)
        ops.gated_rms(o, o, x[:, self.g0:], self.norm, s.heads * s.vdim, self.eps)
        return ops.matmul(o, self.w_out)


class MixtureOfExperts:
    """Top-k routed gated experts plus an optional shared one.  Returns expert rows; the weighted sum rides in the norm behind."""

    def __init__(self, s: MoeSpec, w: Weights, ops: LmOps, width: int):
        self.s, self.ops = s, ops
        W, F = pad64(width), pad64(s.ff)
        self.W, self.F = W, F
        self.router = padded(w.matrix("router", s.experts, width), (s.experts + 15) // 16 * 16, W)
        self.bias = w.vector("router.b", s.experts)
        self.w_in = torch.stack([pair_rows(w.matrix("e%d.gate" % e, s.ff, width), w.matrix("e%d.up" % e, s.ff, width), F, W)
                                 for e in range(s.experts)])
        self.w_out = torch.stack([padded(w.matrix("e%d.down" % e, width, s.ff), W, F) for e in range(s.experts)])
        if s.shared_ff:
            self.FS = pad64(s.shared_ff)
            self.shared_in = pair_rows(w.matrix("shared.gate", s.shared_ff, width), w.matrix("shared.up", s.shared_ff, width), self.FS, W)
            self.shared_out = padded(w.matrix("shared.down", width, s.shared_ff), W, self.FS)

    def __call__(self, h):
        """-> (rows by (token, choice), then by token for the shared expert; (weights, shared) for LmOps.residual_norm)"""
        s, ops, T = self.s, self.ops, h.shape[0]
        wts, order = ops.route(ops.matmul(h, self.router, out_f32=True), self.bias, s.experts, s.top)
        pairs, new = T * s.top, lambda r, c: torch.empty((r, c), dtype=h.dtype, device=h.device)      # noqa: E731
        act, y = new(pairs, self.F), new(pairs + (T if s.shared_ff else 0), self.W)
        up = down = None
        if s.shared_ff:
            act_s = new(T, self.FS)
            up, down = (h, self.shared_in, act_s), (act_s, self.shared_out, y[pairs:])
        ops.grouped(order, T, h, self.w_in, act, False, True, up)
        ops.grouped(order, T, act, self.w_out, y, True, False, down)
        return y, (wts, bool(s.shared_ff))


class Layer:
    def __init__(self, spec: LayerSpec, w: Weights, ops: LmOps, width: int, eps: float, kind: str, mixes: bool):
        W = pad64(width)
        self.is_attention = isinstance(spec.mixer, AttentionSpec)
        self.mixer = (Attention(spec.mixer, w.under("mix."), ops, width, mixes) if self.is_attention else
                      LinearAttention(spec.mixer, w.under("mix."), ops, width, eps))
        self.value_mix = self.is_attention and spec.mixer.value_mix
        self.moe = MixtureOfExperts(spec.moe, w.under("mlp."), ops, width) if spec.moe else None
        self.norms = {n: Norm(w, n, width, W, kind).pair for n in (("norm1", "norm1b", "norm2", "norm2b") if self.moe else
                                                                   ("norm1", "norm1b"))}


class Decoder(EngineModel):
    """A stack of layers with a norm before and after every sublayer over an f32 residual stream.

    One fused launch per sublayer boundary: norm of the sublayer's output, addition, norm for the next sublayer."""

    page_size, attn_rows = PAGE, ATTN_ROWS
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, spec: DecoderSpec, w: Weights, ops: LmOps):
        self.spec, self.ops, self.device, self.dtype, self.vocab = spec, ops, w.device, w.dtype, spec.vocab
        self.W = pad64(spec.width)
        self.embed = padded(w.matrix("embed", spec.vocab, spec.width), spec.vocab, self.W)
        self.head = padded(w.matrix("head", spec.vocab, spec.width), (spec.vocab + 15) // 16 * 16, self.W)
        self.final = Norm(w, "final.norm", spec.width, self.W, spec.norm).pair
        self.layers: List[Layer] = []
        seen = False
        for i, ls in enumerate(spec.layers):
            mixing = isinstance(ls.mixer, AttentionSpec) and ls.mixer.value_mix
            self.layers.append(Layer(ls, w.under("l%d." % i), ops, spec.width, spec.eps, spec.norm, mixing and seen))
            seen = seen or mixing
        shapes = {(l.mixer.s.kv_heads, l.mixer.dv) for l in self.layers if l.value_mix}
        if len(shapes) > 1:
            raise ValueError("layers that mix values need the same kv heads and value size")
        self.tap = None          # called with the residual stream after every layer (tests); None in production

    # ---- what the engine allocates ----
    def kv_shapes(self):
        return [l.mixer.cache_shape() for l in self.layers if l.is_attention]

    def state_shapes(self):
        return [l.mixer.state_shape() for l in self.layers if not l.is_attention]

    def window(self):
        ws = [l.mixer.s.window for l in self.layers if l.is_attention]
        return None if any(x is None for x in ws) else max(ws, default=1)

    def linear_workgroups(self):
        return min((h * dv // 64 for h, _, dv in self.state_shapes()), default=0)

    # ---- one step ----
    def forward(self, b, cache):
        ops, spec, W = self.ops, self.spec, self.W
        T = b.tokens.numel()
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)
        h = torch.empty((T, W), dtype=self.dtype, device=self.device)
        norm = lambda **kw: ops.residual_norm(x, spec.width, spec.norm, spec.eps, **kw)      # noqa: E731
        norm(tokens=b.tokens, embed=self.embed, next=self.layers[0].norms["norm1"], h=h)
        v_first, kv, st = None, iter(cache.kv), iter(cache.state)
        last = len(self.layers) - 1
        out = None
        for i, L in enumerate(self.layers):
            if L.is_attention:
                y, v = L.mixer(h, b, next(kv), v_first)
                if L.value_mix and v_first is None:
                    v_first = v
            else:
                y = L.mixer(h, b, next(st))
            experts, post = None, L.norms["norm1b"]
            if L.moe is not None:
                norm(y=y, post=post, next=L.norms["norm2"], h=h)
                y, experts = L.moe(h)
                post = L.norms["norm2b"]
            if i < last:
                norm(y=y, experts=experts, post=post, next=self.layers[i + 1].norms["norm1"], h=h)
            elif self.tap is not None:
                norm(y=y, experts=experts, post=post)
                y = None
            if self.tap is not None:
                self.tap(i, x[:, :spec.width])
        if b.rows.numel():
            hs = torch.empty((b.rows.numel(), W), dtype=self.dtype, device=self.device)
            norm(y=y, experts=experts if y is not None else None, post=post, next=self.final, h=hs, rows=b.rows, store_x=False)
            out = ops.matmul(hs, self.head, out_f32=True, scale=spec.logit_scale)[:, :self.vocab]
        return out

    def greedy(self, logits):
        return self.ops.argmax(logits, self.vocab)
