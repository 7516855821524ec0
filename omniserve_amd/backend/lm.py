"""ctypes binding of the engine's layer kernels (include/omniserve_lm.h), one library per element type.

`lm_ops(dtype)` loads the library of torch.bfloat16 or torch.float32, building it first when the checkout holds none (after a change
to a source: `python -m omniserve_amd.build`).  There is no CPU fallback: tensors must live on the GPU."""
from __future__ import annotations

import ctypes
import os
import threading

import torch

from .. import _lib

_c = ctypes
_vp, _i, _i64, _f = _c.c_void_p, _c.c_int, _c.c_int64, _c.c_float

ELEM = {torch.bfloat16: "bf16", torch.float32: "f32"}
NORM = {"layer": 0, "rms": 1}
ACT = {None: 0, "silu": 1, "gelu_tanh": 2, "sigmoid": 3}
EPI_ELEM, EPI_F32, EPI_GLU, EPI_GATE = 0, 1, 2, 3
ABI = 3
ATTN_ROWS = 128          # query rows of one prefill tile
PAGE = 64                # tokens per cache page
ROWS_MAX = 64            # up to here a step's products stream the weights
NARROW = 128             # products of so few channels do for any number of rows


class _Part(_c.Structure):
    _fields_ = [("w", _vp), ("x", _vp), ("ldx", _i64), ("y", _vp), ("ldy", _i64), ("n", _i), ("k", _i),
                ("gx", _i64), ("gy", _i64), ("bias", _vp), ("gate", _vp), ("ldg", _i64)]


_PP = _c.POINTER(_Part)
PROTOTYPES = {
    "lm_abi_version": (_i, []),
    "lm_elem_bytes": (_i, []),
    "lm_residual_norm": (_i, [_vp, _i64, _vp, _vp, _f, _vp, _i64, _vp, _vp, _i, _i, _i, _vp, _vp, _vp, _vp, _vp, _i64, _vp, _i, _i, _i, _i, _f, _vp]),
    "lm_gated_rms": (_i, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _i, _i, _i, _f, _vp]),
    "lm_rope_append": (_i, [_vp, _i64, _vp, _i64, _f, _vp, _i, _vp, _vp, _vp, _vp, _i, _i, _i, _i, _i, _vp]),
    "lm_attn_prefill": (_i, [_vp, _i64, _vp, _i64, _i, _i, _vp, _i64, _i, _i, _vp, _i, _vp, _vp, _i, _vp, _i64, _vp, _i64, _f, _i, _i, _i, _i, _i, _vp]),
    "lm_attn_decode": (_i, [_vp, _i64, _vp, _i64, _f, _vp, _i, _vp, _vp, _vp, _vp, _vp, _i, _vp, _i64, _vp, _i64, _vp, _i, _f, _i, _i, _i,
                            _i, _i, _i, _vp]),
    "lm_linear_prefill": (_i, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _i, _i, _i, _vp, _i, _i, _i, _i, _vp]),
    "lm_linear_decode": (_i, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _vp, _i, _i, _i, _i, _i, _vp]),
    "lm_latent_append": (_i, [_vp, _i64, _i64, _vp, _f, _vp, _i, _vp, _vp, _vp, _i, _i, _i, _i, _i, _i, _i, _vp]),
    "lm_gather_pages": (_i, [_vp, _vp, _vp, _i, _i, _vp]),
    "lm_latent_decode": (_i, [_vp, _i64, _i64, _vp, _f, _vp, _i, _vp, _vp, _vp, _vp, _i, _vp, _vp, _vp, _i, _f, _i, _i, _i, _i, _i, _i, _i,
                              _vp]),
    "lm_glu": (_i, [_vp, _i64, _vp, _i64, _vp, _i, _i, _i, _vp]),
    "lm_gated_head_rms": (_i, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _i, _i, _i, _i, _f, _i, _vp]),
    "lm_gla_prefill": (_i, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _vp, _i, _i, _i64, _vp, _vp, _i, _f, _f, _i, _i, _i, _vp]),
    "lm_gla_decode": (_i, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _i64, _vp, _vp, _i, _f, _f, _i64, _vp, _i, _f, _i, _i, _i, _i, _vp]),
    "lm_delta_chunk_rows": (_i, []),
    "lm_delta_mat_elems": (_i64, []),
    "lm_delta_prefill": (_i, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _vp, _vp, _i, _vp, _i, _i, _vp, _i, _f, _f, _i64, _vp, _vp, _vp, _vp,
                              _vp, _vp, _i, _i, _i, _i, _vp]),
    "lm_delta_decode": (_i, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _vp, _vp, _i, _f, _f, _i64, _vp, _vp, _i64, _vp, _i, _f, _i, _i, _i, _i,
                             _i, _vp]),
    "lm_route_scratch_words": (_i64, [_i, _i, _i]),
    "lm_route_max_tiles": (_i, [_i, _i, _i]),
    "lm_route": (_i, [_vp, _i64, _vp, _i, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp]),
    "lm_gemm_rows": (_i, [_PP, _PP, _i, _vp, _vp, _i, _i, _i, _i, _f, _i, _i, _vp]),
    "lm_gemm_tiles": (_i, [_PP, _PP, _i, _vp, _vp, _vp, _i, _i, _i, _i, _f, _i, _i, _vp]),
    "lm_argmax": (_i, [_vp, _vp, _i64, _i, _i, _vp]),
}


def _p(t):
    return None if t is None else t.data_ptr()


def _ld(t):
    return 0 if t is None else t.stride(0)


class LmOps:
    """The kernels of one element type over torch tensors.  Row-major operands may be views with a row stride."""

    def __init__(self, dtype: torch.dtype):
        if dtype not in ELEM:
            raise ValueError("no layer kernels for %s (bfloat16 and float32 have them)" % dtype)
        from .. import build
        self.dtype = dtype
        path = build.lm_lib_path(ELEM[dtype])
        h = _c.CDLL(path if os.path.exists(path) else build.build_lm(ELEM[dtype]))
        for name, (res, args) in PROTOTYPES.items():
            fn = getattr(h, name)
            fn.restype, fn.argtypes = res, args
        if h.lm_abi_version() != ABI or h.lm_elem_bytes() != torch.empty((), dtype=dtype).element_size():
            raise RuntimeError("the layer library does not match its binding: run `python -m omniserve_amd.build --force`")
        self._h = h
        self.delta_chunk = h.lm_delta_chunk_rows()      # tokens per chunk of the delta rule

    def _call(self, name, *args):
        _lib.check(getattr(self._h, name)(*args, _lib.current_stream()), name)

    def residual_norm(self, x, n, kind, eps, *, tokens=None, embed=None, embed_scale=1.0, y=None, y_bias=None, experts=None, post=None,
                      next=None, h=None, rows=None, store_x=True):
        """experts: (pair weights [tokens, top], shared) when y holds expert rows; post / next: (weight, bias or None); h without
        next: the new residual itself."""
        pw, shared = experts if experts is not None else (None, False)
        top = pw.shape[1] if pw is not None else 0
        pairs = pw.numel() if pw is not None else 0
        post, nxt = post or (None, None), next or (None, None)
        self._call("lm_residual_norm", _p(x), _ld(x), _p(tokens), _p(embed), embed_scale, _p(y), _ld(y), _p(y_bias), _p(pw), top, pairs, int(bool(shared)),
                   _p(post[0]), _p(post[1]), _p(nxt[0]), _p(nxt[1]), _p(h), _ld(h), _p(rows),
                   x.shape[0] if rows is None else rows.numel(), n, NORM[kind], int(store_x), eps)

    def gated_rms(self, out, o, gate, w, n, eps):
        self._call("lm_gated_rms", _p(out), _ld(out), _p(o), _ld(o), _p(gate), _ld(gate), _p(w), o.shape[0], o.shape[1], n, eps)

    def rope_append(self, qkv, v_first, lam, freq, pos, slot, kc, vc, heads, kv_heads, dk, dv):
        self._call("lm_rope_append", _p(qkv), _ld(qkv), _p(v_first), _ld(v_first), lam, _p(freq), freq.numel(), _p(pos), _p(slot), _p(kc),
                   _p(vc), qkv.shape[0], heads, kv_heads, dk, dv)

    def attn_prefill(self, q, k, v, bt, entry, tiles, gate, o, scale, window, heads, kv_heads, dk, dv):
        """k, v: cache pools [pages, kv_heads, 64, size], or rows [pages * 64, kv_heads * size] (views with a row stride)"""
        at = lambda t, d: (t.stride(0), t.stride(1), t.stride(2)) if t.dim() == 4 else (PAGE * t.stride(0), d, t.stride(0))      # noqa: E731
        self._call("lm_attn_prefill", _p(q), _ld(q), _p(k), *at(k, dk), _p(v), *at(v, dv), _p(bt), bt.stride(0), _p(entry), _p(tiles), tiles.shape[0], _p(gate),
                   _ld(gate), _p(o), _ld(o), scale, window, heads, kv_heads, dk, dv)

    def attn_decode(self, qkv, v_first, lam, freq, pos, slot, kc, vc, bt, gate, o, part, nsplit, scale, window, heads, kv_heads, dk, dv):
        self._call("lm_attn_decode", _p(qkv), _ld(qkv), _p(v_first), _ld(v_first), lam, _p(freq), freq.numel(), _p(pos), _p(slot), _p(kc),
                   _p(vc), _p(bt), bt.stride(0), _p(gate), _ld(gate), _p(o), _ld(o), _p(part), nsplit, scale, window, qkv.shape[0], heads,
                   kv_heads, dk, dv)

    def linear_prefill(self, x, o, state, seg_state, seg, seg_len, multi, log2_decay, heads, dk, dv, act):
        self._call("lm_linear_prefill", _p(x), _ld(x), _p(o), _ld(o), _p(state), _p(seg_state), _p(seg), seg.shape[0], seg_len, int(multi),
                   _p(log2_decay), heads, dk, dv, ACT[act])

    def linear_decode(self, x, o, state, slot, pos, log2_decay, heads, dk, dv, act):
        self._call("lm_linear_decode", _p(x), _ld(x), _p(o), _ld(o), _p(state), _p(slot), _p(pos), _p(log2_decay), x.shape[0], heads, dk,
                   dv, ACT[act])

    # ---- latent attention: sizes = (heads, query row, first turned column, R, Rp, Tp) ------------------------------
    def latent_append(self, x, src_col, w, eps, freq, pos, slot, cache, sizes):
        self._call("lm_latent_append", _p(x), _ld(x), src_col, _p(w), eps, _p(freq), freq.numel(), _p(pos), _p(slot), _p(cache), x.shape[0],
                   *sizes)

    def gather_pages(self, cache, pages, row):
        out = torch.empty((pages.numel() * PAGE, row), dtype=self.dtype, device=cache.device)
        self._call("lm_gather_pages", _p(out), _p(cache), _p(pages), pages.numel(), row)
        return out

    def latent_decode(self, x, src_col, w, eps, freq, pos, slot, cache, bt, qa, o, part, nsplit, scale, sizes):
        self._call("lm_latent_decode", _p(x), _ld(x), src_col, _p(w), eps, _p(freq), freq.numel(), _p(pos), _p(slot), _p(cache), _p(bt),
                   bt.stride(0), _p(qa), _p(o), _p(part), nsplit, scale, x.shape[0], *sizes)

    # ---- gated recurrences ------------------------------------------------------------------------------------------
    def gated_head_rms(self, out, o, gate, w, heads, dv, n, eps, act):
        self._call("lm_gated_head_rms", _p(out), _ld(out), _p(o), _ld(o), _p(gate), _ld(gate), _p(w), o.shape[0], heads, dv, n, eps, ACT[act])

    def gla_prefill(self, x, o, state, seg_state, seg_decay, seg, multi, low_col, a2, bias, tau, scale, heads, dk, dv):
        self._call("lm_gla_prefill", _p(x), _ld(x), _p(o), _ld(o), _p(state), _p(seg_state), _p(seg_decay), _p(seg), seg.shape[0], int(multi),
                   low_col, _p(a2), _p(bias), a2.shape[1], 1.0 / tau, scale, heads, dk, dv)

    def gla_decode(self, x, o, state, slot, pos, low_col, a2, bias, tau, scale, gate_col, w, n, eps, heads, dk, dv):
        self._call("lm_gla_decode", _p(x), _ld(x), _p(o), _ld(o), _p(state), _p(slot), _p(pos), low_col, _p(a2), _p(bias), a2.shape[1],
                   1.0 / tau, scale, gate_col, _p(w), n, eps, x.shape[0], heads, dk, dv)

    def delta_prefill(self, x, o, state, ring, portions, chunks, seg, multi, conv_w, qk_eps, scale, ab_col, a_log, dt_bias, heads, kv_heads, dk, dv):
        T, n, dev = x.shape[0], chunks.numel(), x.device
        f32 = lambda *s: torch.empty(s, dtype=torch.float32, device=dev)      # noqa: E731
        y = torch.empty((T, conv_w.shape[1]), dtype=self.dtype, device=dev)
        mats = torch.empty((n * heads * self._h.lm_delta_mat_elems(),), dtype=self.dtype, device=dev)
        norms, vecs = f32(T, 2 * kv_heads), f32(n, heads, 4, self.delta_chunk)
        seg_state = f32(seg.shape[0], heads, dk * (dv + dk)) if multi else None
        self._call("lm_delta_prefill", _p(x), _ld(x), _p(o), _ld(o), _p(state), _p(ring), _p(seg_state), _p(portions), _p(chunks), n, _p(seg),
                   seg.shape[0], int(multi), _p(conv_w), conv_w.shape[0], qk_eps, scale, ab_col, _p(a_log), _p(dt_bias), _p(y), _p(norms), _p(mats), _p(vecs), heads,
                   kv_heads, dk, dv)

    def delta_decode(self, x, o, state, ring, slot, pos, conv_w, qk_eps, scale, ab_col, a_log, dt_bias, gate_col, w, n, eps, heads, kv_heads,
                     dk, dv):
        self._call("lm_delta_decode", _p(x), _ld(x), _p(o), _ld(o), _p(state), _p(ring), _p(slot), _p(pos), _p(conv_w), conv_w.shape[0],
                   qk_eps, scale, ab_col, _p(a_log), _p(dt_bias), gate_col, _p(w), n, eps, x.shape[0], heads, kv_heads, dk, dv)

    def argmax(self, z, n):
        out = torch.empty((z.shape[0],), dtype=torch.int64, device=z.device)
        self._call("lm_argmax", _p(out), _p(z), _ld(z), z.shape[0], n)
        return out

    # ---- products ------------------------------------------------------------------------------------------------
    def matmul(self, x, w, out=None, out_f32=False, scale=1.0):
        """x [T, k] w[n, k]^T.  Few rows: the weight-streaming kernel; many: the MFMA tiles for f32 results (the router, the
        output head), the vendor product for plain ones."""
        T, n = x.shape[0], w.shape[0]
        if out is None:
            out = torch.empty((T, n), dtype=torch.float32 if out_f32 else self.dtype, device=x.device)
        if T > ROWS_MAX and not out_f32:
            return torch.mm(x, w.t(), out=out)
        part = _Part(_p(w), _p(x), _ld(x), _p(out), _ld(out), n, w.shape[1])
        epi = EPI_F32 if out_f32 else EPI_ELEM
        if T <= ROWS_MAX or n <= NARROW:
            self._call("lm_gemm_rows", _c.byref(part), None, 1, None, None, T, 0, 1, T, scale, epi, 0)
        else:
            self._call("lm_gemm_tiles", _c.byref(part), None, 1, None, None, None, 0, T, 0, 1, scale, epi, 0)
        return out

    def glu(self, x, w, bias, act):
        """act(x gate^T + bias) * (x up^T + bias); w [2 n, k] (and its bias) in alternating blocks of 16 gate and up channels.  Few
        rows: one launch; many: the vendor product and a row kernel."""
        T, n = x.shape[0], w.shape[0] // 2
        out = torch.empty((T, n), dtype=self.dtype, device=x.device)
        if T <= ROWS_MAX:
            part = _Part(_p(w), _p(x), _ld(x), _p(out), _ld(out), 2 * n, w.shape[1], bias=_p(bias))
            self._call("lm_gemm_rows", _c.byref(part), None, 1, None, None, T, 0, 1, T, 1.0, EPI_GLU, ACT[act])
        else:
            y = self.matmul(x, w)
            self._call("lm_glu", _p(out), _ld(out), _p(y), _ld(y), _p(bias), T, n, ACT[act])
        return out

    def head_products(self, x, w, out, x_step, out_step, gate=None):
        """One matrix per head, w [heads, n, k]: head h reads x from column h * x_step and writes out from column h * out_step;
        gate (laid out like out): times sigmoid(gate)."""
        H, n, k = w.shape
        part = _Part(_p(w), _p(x), _ld(x), _p(out), _ld(out), n, k, gx=x_step, gy=out_step, gate=_p(gate), ldg=_ld(gate))
        T = x.shape[0]
        self._call("lm_gemm_rows", _c.byref(part), None, H, None, None, T, 0, 1, T, 1.0, EPI_ELEM if gate is None else EPI_GATE, 0)
        return out

    def route(self, z, bias, experts, top):
        """-> (weights [T, top], the order of the grouped products)"""
        T, dev = z.shape[0], z.device
        wts = torch.empty((T, top), dtype=torch.float32, device=dev)
        off = torch.empty((experts + 1,), dtype=torch.int32, device=dev)
        perm = torch.empty((T * top,), dtype=torch.int32, device=dev)
        tiles = scratch = None
        max_tiles = 0
        if T > ROWS_MAX:
            max_tiles = self._h.lm_route_max_tiles(T, experts, top)
            tiles = torch.empty((max_tiles, 4), dtype=torch.int32, device=dev)
            scratch = torch.empty((self._h.lm_route_scratch_words(T, experts, top),), dtype=torch.int32, device=dev)
        self._call("lm_route", _p(z), _ld(z), _p(bias), T, experts, top, _p(wts), _p(off), _p(perm), _p(tiles), _p(scratch))
        return wts, (off, perm, tiles, max_tiles, top)

    def grouped(self, order, tokens, x, w, y, x_is_pairs, glu, extra=None):
        """Expert products: w [experts, n, k]; x rows per token or per (token, choice); extra = (x, w, y) of the shared expert."""
        off, perm, tiles, max_tiles, top = order
        a = _Part(_p(w), _p(x), _ld(x), _p(y), _ld(y), w.shape[1], w.shape[2])
        b = None
        if extra is not None:
            b = _Part(_p(extra[1]), _p(extra[0]), _ld(extra[0]), _p(extra[2]), _ld(extra[2]), extra[1].shape[0], extra[1].shape[1])
        pb = None if b is None else _c.byref(b)
        epi, div, rb = (EPI_GLU if glu else EPI_ELEM), (1 if x_is_pairs else top), (tokens if b is not None else 0)
        if tiles is None:
            self._call("lm_gemm_rows", _c.byref(a), pb, w.shape[0], _p(perm), _p(off), 0, rb, div, tokens, 1.0, epi, ACT["silu"])
        else:
            self._call("lm_gemm_tiles", _c.byref(a), pb, w.shape[0], _p(perm), _p(off), _p(tiles), max_tiles, 0, rb, div, 1.0, epi, ACT["silu"])


_ops = {}
_lock = threading.Lock()


def lm_ops(dtype: torch.dtype) -> LmOps:
    with _lock:
        if dtype not in _ops:
            _ops[dtype] = LmOps(dtype)
        return _ops[dtype]
