"""Building blocks of the decoder models the engine serves: specifications (sizes and constants) and the layers that run them on
the kernels of backend/lm.py.

Inner sizes are padded with zeros when the weights are loaded -- the model width and the feed-forward to multiples of 64, every
head to 64, 128 or 256 (192 too for expanded latent keys), a latent to 64, 128, 256 or 512 -- so that the kernels' k loops carry no bounds.  A padded q / k dimension adds zero to every score, a
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
EXPAND_PAGES = 1024          # context pages whose keys and values exist at once (a longer context alone is expanded as a whole)


# ---------------------------------------------------------------------------------------------------------------
# specifications
# ---------------------------------------------------------------------------------------------------------------
@dataclasses.dataclass(frozen=True)
class RotarySpec:
    dims: int                         # leading dimensions of a head that turn
    base: float
    scaling: Optional[dict] = None    # factor, low, high, original: see rope.inverse_frequencies
    pairing: str = "neighbours"       # (2i, 2i + 1) turn together; "halves": (i, i + dims / 2)


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
        if self.rotary is not None and self.rotary.pairing != "neighbours":
            raise ValueError("this attention turns neighbouring pairs")


@dataclasses.dataclass(frozen=True)
class LatentAttentionSpec:
    heads: int
    dim: int                          # unturned query / key dimensions of a head
    vdim: int
    kv_rank: int                      # the latent all heads' keys and values are read from
    rotary: RotarySpec                # all of one more key part, shared by the heads, and of its query parts
    scale: float
    kv_from: Optional[int] = None     # the layer whose latent and turned key part this one attends to

    def __post_init__(self):
        if not self.scale > 0:
            raise ValueError("the score scale must be positive")
        if self.rotary.dims % 2 or self.rotary.dims < 2 or self.rotary.pairing != "halves" or self.rotary.scaling:
            raise ValueError("the shared key part has an even size and turns (i, i + size / 2) together, unscaled")
        if min(self.heads, self.dim, self.vdim, self.kv_rank) < 1:
            raise ValueError("sizes must be positive")


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
class GatedLinearAttentionSpec:
    """S <- diag(alpha) S + k v^T with a low-rank decay per key channel, alpha = sigmoid(W_a2 W_a1 h + b)^(1 / tau)"""
    heads: int
    dim: int
    vdim: int
    tau: float

    def __post_init__(self):
        if not self.tau > 0:
            raise ValueError("tau must be positive")


@dataclasses.dataclass(frozen=True)
class DeltaSpec:
    """Gated delta rule behind short convolutions; query / key heads shared by groups of value heads"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int                         # of the convolutions, the current input included
    unit_eps: float = 1e-6            # q, k: x / sqrt(sum x^2 + unit_eps)

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if self.taps < 1:
            raise ValueError("a convolution sees at least the current input")


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    """down(act(gate h) * up h), every projection with a bias"""
    ff: int
    act: str = "gelu_tanh"

    def __post_init__(self):
        if self.act not in ("silu", "gelu_tanh"):
            raise ValueError("unknown activation %r" % self.act)


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
    mixer: object                     # one of the mixers' specs above
    ff: object                        # MoeSpec, DenseSpec or None


@dataclasses.dataclass(frozen=True)
class DecoderSpec:
    vocab: int
    width: int
    layers: Tuple[LayerSpec, ...]
    eps: float
    norm: str = "layer"               # "layer" (weight and bias) or "rms" (weight)
    logit_scale: float = 1.0
    placement: str = "around"         # norms before and after every sublayer (norm1 / norm1b, norm2 / norm2b), or only
                                      # "after" it (norm1, norm2): the sublayers then read the residual itself
    embed_scale: float = 1.0

    def __post_init__(self):
        if self.norm not in ("layer", "rms") or self.placement not in ("around", "after"):
            raise ValueError("unknown norm %r / %r" % (self.norm, self.placement))
        for i, l in enumerate(self.layers):
            j = getattr(l.mixer, "kv_from", None)
            if j is None:
                continue
            src = self.layers[j].mixer if 0 <= j < i else None
            if not isinstance(src, LatentAttentionSpec) or src.kv_from is not None or (src.kv_rank, src.rotary) != (l.mixer.kv_rank, l.mixer.rotary):
                raise ValueError("layer %d cannot read the latents of layer %d" % (i, j))


# ---------------------------------------------------------------------------------------------------------------
# padding
# ---------------------------------------------------------------------------------------------------------------
def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def pad_to(n: int, *sizes) -> int:
    for p in sizes:
        if n <= p:
            return p
    raise ValueError("size %d is larger than the kernels' %d" % (n, sizes[-1]))


def pad_head(n: int) -> int:
    return pad_to(n, 64, 128, 256)


def padded(t: torch.Tensor, *sizes) -> torch.Tensor:
    """t in the corner of a zero tensor of these sizes."""
    if tuple(t.shape) == tuple(sizes):
        return t.contiguous()
    out = t.new_zeros(sizes)
    out[tuple(slice(0, s) for s in t.shape)] = t
    return out


def pad_out_heads(w, heads, dim, width, size=None):
    """[heads * dim, in] -> [heads * size, width], size: pad_head(dim) unless given"""
    size = size or pad_head(dim)
    return padded(w.reshape(heads, dim, w.shape[1]), heads, size, width).reshape(heads * size, width)


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

    def rows(self, name):
        """first size of a tensor that only the checkpoint knows"""
        if self.prefix + name not in self.state:
            raise RuntimeError("the checkpoint lacks tensor %s" % (self.prefix + name))
        return int(self.state[self.prefix + name].shape[0])

    def leftovers(self, optional=()):
        return sorted(k for k in self.state if k not in self.used and not any(k.endswith(o) for o in optional))


# ---------------------------------------------------------------------------------------------------------------
# layers
# ---------------------------------------------------------------------------------------------------------------
class Norm:
    def __init__(self, w: Weights, name: str, width: int, size: int, kind: str):
        self.pair = (w.vector(name, width, size), w.vector(name + ".b", width, size) if kind == "layer" else None)


class Mixer:
    """What a mixer asks of the cache and the batch."""
    segment_workgroups = 0            # workgroups one segment of a prompt gives to the layer (0: it does not use segments)

    def cache_shape(self):
        """(kv heads, key size, value size) of its pages, None without"""
        return None

    def state_shapes(self):
        return []


class Attention(Mixer):
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


class LinearAttention(Mixer):
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

        self.segment_workgroups = H * self.dv // 64

    def state_shapes(self):
        return [(self.s.heads, self.dk, self.dv)]

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


class LatentAttention(Mixer):
    """Softmax attention whose keys and values are read from one latent per token: the cache holds the normed latent and a turned key
    part for all heads, own or another layer's.

    Prompts expand the context's rows into keys and values of every head by one product -- its matrix holds an identity for the turned
    part -- and run the attention kernel on them.  Single tokens stay in the latent space: W_uk^T q scores against the rows themselves
    and W_uv is applied to the weighted sum of latents."""

    def __init__(self, s: LatentAttentionSpec, w: Weights, ops: LmOps, width: int, eps: float):
        self.s, self.ops, self.eps = s, ops, eps
        H, W, R, rot = s.heads, pad64(width), s.kv_rank, s.rotary.dims
        self.rot0 = (s.dim + 7) // 8 * 8                      # a query row: unturned part, turned part from rot0 on, zeros
        self.dk, self.dv = pad_to(self.rot0 + rot, 64, 128, 192, 256), pad_head(s.vdim)
        self.Rp, self.Tp = pad_to(R, 64, 128, 256, 512), pad_to(rot, 64, 128)
        self.row = self.Rp + self.Tp
        q = w.matrix("q", H * (s.dim + rot), width).reshape(H, s.dim + rot, width)
        qp = q.new_zeros((H, self.dk, W))
        qp[:, :s.dim, :width], qp[:, self.rot0:self.rot0 + rot, :width] = q[:, :s.dim], q[:, s.dim:]
        parts = [qp.reshape(H * self.dk, W), pad_out_heads(w.matrix("g", H * s.vdim, width), H, s.vdim, W)]
        self.g0, self.src = H * self.dk, -1
        self.norm = None
        if s.kv_from is None:
            self.src = self.g0 + H * self.dv
            d = w.matrix("dkv", R + rot, width)
            parts += [padded(d[:R], self.Rp, W), padded(d[R:], self.Tp, W)]
            self.norm = w.vector("dkv.norm", R, self.Rp)
        self.w_in = torch.cat(parts)
        self.w_out = pad_in_heads(w.matrix("o", width, H * s.vdim), H, s.vdim, W)
        uk, uv = w.matrix("uk", H * s.dim, R).reshape(H, s.dim, R), w.matrix("uv", H * s.vdim, R).reshape(H, s.vdim, R)
        self.w_score = padded(uk.transpose(1, 2), H, self.Rp, pad64(s.dim))
        self.w_value = padded(uv, H, self.dv, self.Rp)
        k = uk.new_zeros((H, self.dk, self.row))
        k[:, :s.dim, :R] = uk
        k[:, self.rot0:self.rot0 + rot, self.Rp:self.Rp + rot] = torch.eye(rot, dtype=uk.dtype, device=uk.device)
        self.w_kv = torch.cat([k.reshape(H * self.dk, self.row), padded(uv, H, self.dv, self.row).reshape(H * self.dv, self.row)])
        self.freq = torch.tensor(inverse_frequencies(rot, s.rotary.base), dtype=torch.float64).to(device=w.device, dtype=torch.float32)
        self.sizes = (H, self.dk, self.rot0, R, self.Rp, self.Tp)

    def cache_shape(self):
        return (1, self.row, 0) if self.s.kv_from is None else None

    def __call__(self, h, b, pool, contexts):
        """pool: the rows' pages, its own or another layer's; contexts: what layers over the same pool have gathered in this step"""
        s, ops, n, H = self.s, self.ops, b.n_prompt, self.s.heads
        x = ops.matmul(h, self.w_in)
        new = lambda *shape: torch.empty(shape, dtype=h.dtype, device=h.device)      # noqa: E731
        o = new(h.shape[0], H * self.dv)
        if n:
            ops.latent_append(x[:n], self.src, self.norm, self.eps, self.freq, b.pos, b.kv_slot, pool, self.sizes)
            for page0, pages, tile0, tiles in b.expansions:
                if page0 not in contexts:
                    contexts[page0] = ops.gather_pages(pool, b.context_pages[page0:page0 + pages], self.row)
                kv = ops.matmul(contexts[page0], self.w_kv)
                ops.attn_prefill(x[:n], kv[:, :H * self.dk], kv[:, H * self.dk:], b.context_table, b.entry, b.attn_tiles[tile0:tile0 + tiles],
                                 x[:n, self.g0:], o[:n], s.scale, NO_WINDOW, H, H, self.dk, self.dv)
        if b.n_decode:
            B, xd = b.n_decode, x[n:]
            qa = ops.head_products(xd, self.w_score, new(B, H * self.Rp), self.dk, self.Rp)
            lat, nsplit, part = new(B, H * self.Rp), self.splits(b), None
            if nsplit > 1:
                part = torch.empty((B * H * nsplit * (self.Rp + 2),), dtype=torch.float32, device=h.device)
            ops.latent_decode(xd, self.src, self.norm, self.eps, self.freq, b.pos[n:], b.kv_slot[n:], pool, b.block_table[b.n_entries:], qa, lat,
                              part, nsplit, s.scale, self.sizes)
            ops.head_products(lat, self.w_value, o[n:], self.Rp, self.dv, gate=xd[:, self.g0:])
        return ops.matmul(o, self.w_out)

    def splits(self, b) -> int:
        """Parts of the keys per (sequence, 32 heads): a workgroup per CU, two if each gets 1024 keys; at least 256 keys each (a part
        leaves a latent of f32 per head)."""
        groups, keys = max(b.n_decode * ((self.s.heads + 31) // 32), 1), b.max_context
        return max(1, min(max(256 // groups, min(512 // groups, keys // 1024)), keys // 256, 64))


class GatedLinearAttention(Mixer):
    """Linear attention with a decay per key channel; every head's output normed on its own and gated with silu."""

    def __init__(self, s: GatedLinearAttentionSpec, w: Weights, ops: LmOps, width: int, eps: float):
        self.s, self.ops, self.eps = s, ops, eps
        H, W, rank = s.heads, pad64(width), w.rows("a1")
        self.dk, self.dv, low = pad_head(s.dim), pad_head(s.vdim), pad64(rank)
        self.w_in = torch.cat([pad_out_heads(w.matrix("q", H * s.dim, width), H, s.dim, W),
                               pad_out_heads(w.matrix("k", H * s.dim, width), H, s.dim, W),
                               pad_out_heads(w.matrix("v", H * s.vdim, width), H, s.vdim, W),
                               pad_out_heads(w.matrix("g", H * s.vdim, width), H, s.vdim, W), padded(w.matrix("a1", rank, width), low, W)])
        self.g0 = 2 * H * self.dk + H * self.dv
        self.low0 = self.g0 + H * self.dv
        self.a2 = pad_out_heads(w.matrix("a2", H * s.dim, rank), H, s.dim, low)
        bias = torch.full((H, self.dk), 60.0, dtype=torch.float32, device=w.device)      # padded channels do not decay
        bias[:, :s.dim] = w.vector("a2.b", H * s.dim).view(H, s.dim)
        self.bias = bias.view(-1)
        self.w_out = pad_in_heads(w.matrix("o", width, H * s.vdim), H, s.vdim, W)
        self.norm = w.vector("norm", s.vdim, self.dv)
        self.segment_workgroups = max(1, H * self.dv // 128)

    def state_shapes(self):
        return [(self.s.heads, self.dk, self.dv)]

    def __call__(self, h, b, state):
        s, ops, n = self.s, self.ops, b.n_prompt
        x = ops.matmul(h, self.w_in)
        o = torch.empty((h.shape[0], s.heads * self.dv), dtype=h.dtype, device=h.device)
        size, scale = (s.heads, self.dk, self.dv), s.dim ** -0.5
        if n:
            seg_state = seg_decay = None
            if b.multi_segment:
                f32 = lambda *shape: torch.empty(shape, dtype=torch.float32, device=h.device)      # noqa: E731
                seg_state, seg_decay = f32(b.segments.shape[0], *size), f32(b.segments.shape[0], s.heads, self.dk)
            ops.gla_prefill(x[:n], o[:n], state, seg_state, seg_decay, b.segments, b.multi_segment, self.low0, self.a2, self.bias, s.tau, scale,
                            *size)
            ops.gated_head_rms(o[:n], o[:n], x[:n, self.g0:], self.norm, s.heads, self.dv, s.vdim, self.eps, "silu")
        if b.n_decode:
            ops.gla_decode(x[n:], o[n:], state, b.state_slot, b.pos[n:], self.low0, self.a2, self.bias, s.tau, scale, self.g0, self.norm,
                           s.vdim, self.eps, *size)
        return ops.matmul(o, self.w_out)


class DeltaRule(Mixer):
    """Gated delta rule behind short convolutions; every head's output normed on its own and gated with silu."""

    def __init__(self, s: DeltaSpec, w: Weights, ops: LmOps, width: int, eps: float):
        self.s, self.ops, self.eps = s, ops, eps
        H, G, W = s.heads, s.kv_heads, pad64(width)
        self.dk, self.dv = pad_head(s.dim), pad_head(s.vdim)
        gates = torch.cat([w.matrix("a", H, width), w.matrix("b", H, width)])
        self.w_in = torch.cat([pad_out_heads(w.matrix("q", G * s.dim, width), G, s.dim, W),
                               pad_out_heads(w.matrix("k", G * s.dim, width), G, s.dim, W),
                               pad_out_heads(w.matrix("v", H * s.vdim, width), H, s.vdim, W),
                               pad_out_heads(w.matrix("g", H * s.vdim, width), H, s.vdim, W), padded(gates, pad64(2 * H), W)])
        self.g0 = 2 * G * self.dk + H * self.dv
        self.ab0 = self.g0 + H * self.dv
        taps = [pad_out_heads(w.matrix(n + ".conv", heads * size, s.taps).float(), heads, size, s.taps)
                for n, heads, size in (("q", G, s.dim), ("k", G, s.dim), ("v", H, s.vdim))]
        self.conv = torch.cat(taps).t().contiguous()          # [taps, channels]
        self.a_log, self.dt_bias = w.vector("A_log", H), w.vector("dt_bias", H)
        self.w_out = pad_in_heads(w.matrix("o", width, H * s.vdim), H, s.vdim, W)
        self.norm = w.vector("norm", s.vdim, self.dv)
        self.segment_workgroups = H * self.dv // 64

    def state_shapes(self):
        return [(self.s.heads, self.dk, self.dv), (self.s.taps, self.g0)]

    def __call__(self, h, b, state, ring):
        s, ops, n = self.s, self.ops, b.n_prompt
        x = ops.matmul(h, self.w_in)
        o = torch.empty((h.shape[0], s.heads * self.dv), dtype=h.dtype, device=h.device)
        rule = (self.conv, s.unit_eps, s.dim ** -0.5, self.ab0, self.a_log, self.dt_bias)
        size = (s.heads, s.kv_heads, self.dk, self.dv)
        if n:
            ops.delta_prefill(x[:n], o[:n], state, ring, b.portions, b.chunks, b.segments, b.multi_segment, *rule, *size)
            ops.gated_head_rms(o[:n], o[:n], x[:n, self.g0:], self.norm, s.heads, self.dv, s.vdim, self.eps, "silu")
        if b.n_decode:
            ops.delta_decode(x[n:], o[n:], state, ring, b.state_slot, b.pos[n:], *rule, self.g0, self.norm, s.vdim, self.eps, *size)
        return ops.matmul(o, self.w_out)


class Dense:
    """Gated feed-forward with biases; the last one rides in the residual kernel behind."""

    def __init__(self, s: DenseSpec, w: Weights, ops: LmOps, width: int):
        self.s, self.ops = s, ops
        W, F = pad64(width), pad64(s.ff)
        self.w_in = pair_rows(w.matrix("gate", s.ff, width), w.matrix("up", s.ff, width), F, W)
        self.b_in = pair_rows(w.vector("gate.b", s.ff)[:, None], w.vector("up.b", s.ff)[:, None], F, 1).reshape(-1).contiguous()
        self.w_out = padded(w.matrix("down", width, s.ff), W, F)
        self.b_out = w.vector("down.b", width, W)

    def __call__(self, h):
        """-> (rows without the last bias, arguments of LmOps.residual_norm that add it)"""
        return self.ops.matmul(self.ops.glu(h, self.w_in, self.b_in, self.s.act), self.w_out), {"y_bias": self.b_out}


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
        """-> (rows by (token, choice), then by token for the shared expert; arguments of LmOps.residual_norm that sum them)"""
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
        return y, {"experts": (wts, bool(s.shared_ff))}


MIXERS = {LatentAttentionSpec: LatentAttention, LinearAttentionSpec: LinearAttention, GatedLinearAttentionSpec: GatedLinearAttention,
          DeltaSpec: DeltaRule}
FEED_FORWARDS = {MoeSpec: MixtureOfExperts, DenseSpec: Dense}


class Layer:
    def __init__(self, spec: LayerSpec, w: Weights, ops: LmOps, model: DecoderSpec, mixes: bool):
        width, eps = model.width, model.eps
        m = w.under("mix.")
        self.mixer = (Attention(spec.mixer, m, ops, width, mixes) if isinstance(spec.mixer, AttentionSpec) else
                      MIXERS[type(spec.mixer)](spec.mixer, m, ops, width, eps))
        self.value_mix = getattr(spec.mixer, "value_mix", False)
        self.ff = FEED_FORWARDS[type(spec.ff)](spec.ff, w.under("mlp."), ops, width) if spec.ff else None
        # norms before / after the mixer and the feed-forward
        norm = lambda n: Norm(w, n, width, pad64(width), model.norm).pair      # noqa: E731
        names = {"around": ("norm1", "norm1b", "norm2", "norm2b"), "after": (None, "norm1", None, "norm2")}[model.placement]
        self.pre, self.post, self.ff_pre, self.ff_post = [n and (i < 2 or self.ff is not None) and norm(n) or None
                                                          for i, n in enumerate(names)]


class Decoder(EngineModel):
    """A stack of layers with norms around or after every sublayer over an f32 residual stream.

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
        seen, self._kv, self._state, pools, states = False, [], [], 0, 0      # a layer's page pool, its slice of the states
        for i, ls in enumerate(spec.layers):
            mixing = isinstance(ls.mixer, AttentionSpec) and ls.mixer.value_mix
            L = Layer(ls, w.under("l%d." % i), ops, spec, mixing and seen)
            self.layers.append(L)
            seen = seen or mixing
            source = getattr(ls.mixer, "kv_from", None)
            own = L.mixer.cache_shape() is not None
            self._kv.append(self._kv[source] if source is not None else pools if own else None)
            pools += own
            n = len(L.mixer.state_shapes())
            self._state.append(slice(states, states + n))
            states += n
        shapes = {(l.mixer.s.kv_heads, l.mixer.dv) for l in self.layers if l.value_mix}
        if len(shapes) > 1:
            raise ValueError("layers that mix values need the same kv heads and value size")
        kinds = {type(l.mixer) for l in self.layers}
        self.min_segments = 3 if kinds & {GatedLinearAttention, DeltaRule} else 1
        self.chunk_rows = ops.delta_chunk if DeltaRule in kinds else 0
        self.expand_pages = EXPAND_PAGES if LatentAttention in kinds else 0
        self.tap = None          # called with the residual stream after every layer (tests); None in production

    # ---- what the engine allocates ----
    def kv_shapes(self):
        return [s for s in (l.mixer.cache_shape() for l in self.layers) if s is not None]

    def state_shapes(self):
        return [s for l in self.layers for s in l.mixer.state_shapes()]

    def window(self):
        ws = [getattr(l.mixer.s, "window", None) for l, kv in zip(self.layers, self._kv) if kv is not None]
        return None if any(x is None for x in ws) else max(ws, default=1)

    def linear_workgroups(self):
        return min((l.mixer.segment_workgroups for l in self.layers if l.mixer.segment_workgroups), default=0)

    # ---- one step ----
    def forward(self, b, cache):
        ops, spec, W = self.ops, self.spec, self.W
        T = b.tokens.numel()
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)
        h = torch.empty((T, W), dtype=self.dtype, device=self.device)
        norm = lambda **kw: ops.residual_norm(x, spec.width, spec.norm, spec.eps, **kw)      # noqa: E731
        norm(tokens=b.tokens, embed=self.embed, embed_scale=spec.embed_scale, next=self.layers[0].pre, h=h)
        v_first, contexts = None, {}
        last = len(self.layers) - 1
        out = None
        for i, L in enumerate(self.layers):
            kv = self._kv[i]
            if isinstance(L.mixer, Attention):
                y, v = L.mixer(h, b, cache.kv[kv], v_first)
                if L.value_mix and v_first is None:
                    v_first = v
            elif isinstance(L.mixer, LatentAttention):
                y = L.mixer(h, b, cache.kv[kv][0], contexts.setdefault(kv, {}))
            else:
                y = L.mixer(h, b, *cache.state[self._state[i]])
            form, post = {}, L.post
            if L.ff is not None:
                norm(y=y, post=post, next=L.ff_pre, h=h)
                y, form = L.ff(h)
                post = L.ff_post
            if i < last:
                norm(y=y, post=post, next=self.layers[i + 1].pre, h=h, **form)
            elif self.tap is not None:
                norm(y=y, post=post, **form)
                y, form = None, {}
            if self.tap is not None:
                self.tap(i, x[:, :spec.width])
        if b.rows.numel():
            hs = torch.empty((b.rows.numel(), W), dtype=self.dtype, device=self.device)
            norm(y=y, post=post, next=self.final, h=hs, rows=b.rows, store_x=False, **form)
            out = ops.matmul(hs, self.head, out_f32=True, scale=spec.logit_scale)[:, :self.vocab]
        return out

    def greedy(self, logits):
        return self.ops.argmax(logits, self.vocab)
