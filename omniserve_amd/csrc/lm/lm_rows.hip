// Row kernels: residual + norms, the gated norm behind a recurrent mixer, rotation + value mixing + cache append, arg-max.
// One workgroup per token; the row stays in registers between the reductions.
#include "lm_common.h"
#include "omniserve_lm.h"

namespace lm {

constexpr int ROW_THREADS = 256;

template <int TH>
struct Row {      // workgroup-wide sums
  float* red;     // [2][TH / 64]
  int phase = 0;
  __device__ __forceinline__ float sum(float v) {
    v = wave_sum(v);
    float* r = red + TH / 64 * (phase & 1);      // two areas in turn: one barrier per sum
    ++phase;
    if ((threadIdx.x & 63) == 0) r[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < TH / 64; i += 4) t += (r[i] + r[i + 1]) + (r[i + 2] + r[i + 3]);
    return t;
  }
};

// v (columns 4 * (TH i + tid) .. + 3, zero from n on) -> normalised in place; kind 0: layer norm, 1: RMS norm
template <int TH, int NV>
__device__ __forceinline__ void normalise(f32x4 (&v)[NV], Row<TH>& row, int n, int kind, float eps, const float* w, const float* b) {
  float mean = 0.f;
  if (kind == LM_NORM_LAYER) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) s += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);
    mean = row.sum(s) / (float)n;
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (TH * i + (int)threadIdx.x);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[i][e] = c + e < n ? v[i][e] - mean : 0.f;
      ss += v[i][e] * v[i][e];
    }
  }
  const float r = 1.0f / sqrtf(row.sum(ss) / (float)n + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (TH * i + (int)threadIdx.x);
    if (c >= n) continue;
    const f32x4 ww = *(const f32x4*)(w + c);
    f32x4 bb = zero4();
    if (b) bb = *(const f32x4*)(b + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i][e] = c + e < n ? v[i][e] * r * ww[e] + bb[e] : 0.f;
  }
}

struct ResidualArgs {
  float* x; int64_t ldx;                     // residual stream
  const int* tokens; const elem_t* embed;    // tokens: the residual starts as these rows of the table [vocab][ldx] ...
  float embed_scale;                         // ... times this
  const elem_t* y; int64_t ldy;              // sublayer output (or null): added to the residual
  const float* y_bias;                       // added to y (or null)
  const float* pair_w; int top, pairs0, shared;   // top > 0: y holds expert outputs by (token, choice), see moe_sum
  const float *post_w, *post_b;              // norm of the sublayer output before it is added (or null)
  const float *next_w, *next_b;              // norm of the new residual for the next sublayer (or null: as it is) -> h
  elem_t* h; int64_t ldh;
  const int* rows;                           // row r of the launch works on token rows[r] (or null: r) and writes h[r]
  int n, kind, store_x;
  float eps;
};

template <int TH, int NV>
__global__ __launch_bounds__(TH) void residual_norm_kernel(ResidualArgs p) {
  __shared__ float red[2 * TH / 64];
  Row<TH> row{red};
  const int r = blockIdx.x, t = p.rows ? p.rows[r] : r, tid = threadIdx.x;
  f32x4 x[NV], y[NV];
  float* xr = p.x + (int64_t)t * p.ldx;
  const elem_t* er = p.tokens ? p.embed + (int64_t)p.tokens[t] * p.ldx : nullptr;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (TH * i + tid);
    x[i] = y[i] = zero4();
    if (c >= p.n) continue;
    x[i] = er ? p.embed_scale * from_quad(*(const quad_t*)(er + c)) : *(const f32x4*)(xr + c);
  }
  if (p.y) {
    if (p.top > 0) {      // weighted sum of the chosen experts' rows (+ the shared expert's)
      const int64_t p0 = (int64_t)t * p.top;
      constexpr int B = NV >= 8 ? 1 : NV >= 4 ? 2 : 4;      // rows in flight
      for (int k0 = 0; k0 < p.top; k0 += B) {
        quad_t v[B][NV];
        float w[B];
#pragma unroll
        for (int b = 0; b < B; ++b) {
          const int k = min(k0 + b, p.top - 1);
          w[b] = k0 + b < p.top ? p.pair_w[p0 + k] : 0.f;
          const elem_t* yr = p.y + (p0 + k) * p.ldy;
#pragma unroll
          for (int i = 0; i < NV; ++i) {
            const int c = 4 * (TH * i + tid);
            v[b][i] = c < p.n ? *(const quad_t*)(yr + c) : to_quad(zero4());
          }
        }
#pragma unroll
        for (int b = 0; b < B; ++b)
#pragma unroll
          for (int i = 0; i < NV; ++i) y[i] += w[b] * from_quad(v[b][i]);
      }
    }
    if (p.top == 0 || p.shared) {
      const elem_t* yr = p.y + (int64_t)(p.top > 0 ? p.pairs0 + t : t) * p.ldy;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = 4 * (TH * i + tid);
        if (c < p.n) y[i] += from_quad(*(const quad_t*)(yr + c));
      }
    }
    if (p.y_bias) {
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = 4 * (TH * i + tid);
        if (c < p.n) y[i] += *(const f32x4*)(p.y_bias + c);
      }
    }
    if (p.post_w) normalise<TH, NV>(y, row, p.n, p.kind, p.eps, p.post_w, p.post_b);
#pragma unroll
    for (int i = 0; i < NV; ++i) x[i] += y[i];
  }
  if (p.store_x) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = 4 * (TH * i + tid);
      if (c < p.ldx) *(f32x4*)(xr + c) = x[i];
    }
  }
  if (!p.h) return;
  if (p.next_w) normalise<TH, NV>(x, row, p.n, p.kind, p.eps, p.next_w, p.next_b);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (TH * i + tid);
    if (c < p.ldh) *(quad_t*)(p.h + (int64_t)r * p.ldh + c) = to_quad(x[i]);
  }
}

// out = rms_norm(o over its n real columns) * w * sigmoid(gate); padded columns of o, w are zero
template <int NV>
__global__ __launch_bounds__(ROW_THREADS) void gated_rms_kernel(elem_t* out, int64_t ldo, const elem_t* o, int64_t ldi,
                                                                const elem_t* gate, int64_t ldg, const float* w, int cols, int n,
                                                                float eps) {
  __shared__ float red[8];
  Row<ROW_THREADS> row{red};
  const int t = blockIdx.x, tid = threadIdx.x;
  f32x4 v[NV];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (ROW_THREADS * i + tid);
    v[i] = c < cols ? from_quad(*(const quad_t*)(o + (int64_t)t * ldi + c)) : zero4();
    ss += (v[i][0] * v[i][0] + v[i][1] * v[i][1]) + (v[i][2] * v[i][2] + v[i][3] * v[i][3]);
  }
  const float r = 1.0f / sqrtf(row.sum(ss) / (float)n + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (ROW_THREADS * i + tid);
    if (c >= cols) continue;
    const f32x4 g = from_quad(*(const quad_t*)(gate + (int64_t)t * ldg + c)), ww = *(const f32x4*)(w + c);
    f32x4 y;
#pragma unroll
    for (int e = 0; e < 4; ++e) y[e] = v[i][e] * r * ww[e] * sigmoid(g[e]);
    *(quad_t*)(out + (int64_t)t * ldo + c) = to_quad(y);
  }
}

// Per head: out = rms_norm(o over n of dv columns) * w * act(gate).  dv / 4 lanes per head.
__global__ __launch_bounds__(ROW_THREADS) void gated_head_rms_kernel(elem_t* out, int64_t ldo, const elem_t* o, int64_t ldi,
                                                                     const elem_t* gate, int64_t ldg, const float* w, int cols, int dv,
                                                                     int n, float eps, int act) {
  const int t = blockIdx.x, lanes = dv / 4;
  for (int c = 4 * (int)threadIdx.x; c < cols; c += 4 * ROW_THREADS) {
    const f32x4 v = from_quad(*(const quad_t*)(o + (int64_t)t * ldi + c)), g = from_quad(*(const quad_t*)(gate + (int64_t)t * ldg + c));
    float ss = (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);      // (padded columns hold zeros)
    for (int m = lanes >> 1; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
    const float r = 1.0f / sqrtf(ss / (float)n + eps);
    const f32x4 ww = *(const f32x4*)(w + c % dv);
    f32x4 y;
#pragma unroll
    for (int e = 0; e < 4; ++e) y[e] = v[e] * r * ww[e] * (act == LM_ACT_SILU ? silu(g[e]) : sigmoid(g[e]));
    *(quad_t*)(out + (int64_t)t * ldo + c) = to_quad(y);
  }
}

// gated unit of rows in alternating blocks of 16 gate and 16 up channels; a thread's channels of GLU_ROWS rows
constexpr int GLU_ROWS = 16;

__global__ __launch_bounds__(ROW_THREADS) void glu_kernel(elem_t* out, int64_t ldo, const elem_t* x, int64_t ldx, const float* bias, int rows,
                                                          int n, int act) {
  const int c = FR * (int)(blockIdx.x * ROW_THREADS + threadIdx.x), s = 32 * (c >> 4) + (c & 15);
  if (c >= n) return;
  float bg[FR], bu[FR];
#pragma unroll
  for (int e = 0; e < FR; ++e) {
    bg[e] = bias ? bias[s + e] : 0.f;
    bu[e] = bias ? bias[s + 16 + e] : 0.f;
  }
  const int64_t t0 = (int64_t)GLU_ROWS * blockIdx.y, t1 = t0 + GLU_ROWS < rows ? t0 + GLU_ROWS : rows;
  constexpr int B = 4;      // rows in flight
  for (int64_t t = t0; t < t1; t += B) {
    frag_t g[B], u[B];
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const elem_t* xr = x + (t + b < t1 ? t + b : t1 - 1) * ldx + s;
      g[b] = *(const frag_t*)xr;
      u[b] = *(const frag_t*)(xr + 16);
    }
#pragma unroll
    for (int b = 0; b < B; ++b) {
      if (t + b >= t1) break;
      frag_t r;
#pragma unroll
      for (int e = 0; e < FR; ++e) {
        const float a = (float)g[b][e] + bg[e];
        r[e] = (elem_t)((act == LM_ACT_GELU_TANH ? gelu_tanh(a) : silu(a)) * ((float)u[b][e] + bu[e]));
      }
      *(frag_t*)(out + (t + b) * ldo + c) = r;
    }
  }
}

// q and k of a projection row turned by their position (pairs (2i, 2i+1) of the first 2 * half dimensions), values mixed with
// the first mixing layer's; k and v go to the cache page, q stays in place.
struct RopeArgs {
  elem_t* qkv; int64_t ld;              // row: q [H][dk], k [G][dk], v [G][dv]
  const elem_t* v_first; int64_t ldv;   // unmixed values of the first mixing layer ([G][dv] of the same tokens) or null
  float lambda;
  const float* freq; int half;          // rotation per position of each pair
  const int* pos; const int* slot;      // slot = page * 64 + offset
  elem_t *kc, *vc;                      // [pages][G][64][dk | dv]
  int H, G, dk, dv;
};

__global__ __launch_bounds__(ROW_THREADS) void rope_append_kernel(RopeArgs p) {
  __shared__ f32x2 cs[256];
  const int t = blockIdx.x, tid = threadIdx.x;
  const int slot = p.slot[t];
  for (int i = tid; i < p.half; i += ROW_THREADS) {
    float s, c;
    sincosf((float)p.pos[t] * p.freq[i], &s, &c);
    cs[i] = (f32x2){c, s};
  }
  __syncthreads();
  elem_t* row = p.qkv + (int64_t)t * p.ld;
  const int cpr = p.dk / FR;       // chunks per head
  for (int i = tid; i < (p.H + p.G) * cpr; i += ROW_THREADS) {
    const int head = i / cpr, d = (i - head * cpr) * FR;
    frag_t v = *(const frag_t*)(row + (int64_t)head * p.dk + d);
#pragma unroll
    for (int e = 0; e < FR; e += 2) {
      const int pr = (d + e) >> 1;
      if (pr < p.half) {
        const float a = (float)v[e], b = (float)v[e + 1];
        v[e] = (elem_t)(a * cs[pr][0] - b * cs[pr][1]);
        v[e + 1] = (elem_t)(b * cs[pr][0] + a * cs[pr][1]);
      }
    }
    if (head < p.H) {
      *(frag_t*)(row + (int64_t)head * p.dk + d) = v;
    } else if (slot >= 0) {
      const int64_t page = slot / PAGE;
      *(frag_t*)(p.kc + ((page * p.G + head - p.H) * PAGE + slot % PAGE) * p.dk + d) = v;
    }
  }
  if (slot < 0) return;
  const int vpr = p.dv / FR;
  const elem_t* vrow = row + (int64_t)(p.H + p.G) * p.dk;
  for (int i = tid; i < p.G * vpr; i += ROW_THREADS) {
    const int head = i / vpr, d = (i - head * vpr) * FR;
    frag_t v = *(const frag_t*)(vrow + (int64_t)head * p.dv + d);
    if (p.v_first) {
      const frag_t f = *(const frag_t*)(p.v_first + (int64_t)t * p.ldv + (int64_t)head * p.dv + d);
#pragma unroll
      for (int e = 0; e < FR; ++e) v[e] = (elem_t)((1.0f - p.lambda) * (float)v[e] + p.lambda * (float)f[e]);
    }
    const int64_t page = slot / PAGE;
    *(frag_t*)(p.vc + ((page * p.G + head) * PAGE + slot % PAGE) * p.dv + d) = v;
  }
}

// first index of the largest value of each row
__global__ __launch_bounds__(1024) void argmax_kernel(int64_t* out, const float* z, int64_t ld, int n) {
  __shared__ float bv[16];
  __shared__ int bi[16];
  const float* r = z + (int64_t)blockIdx.x * ld;
  float best = -INFINITY;
  int at = 0x7fffffff;
  for (int i = threadIdx.x; i < n; i += 1024) {
    const float v = r[i];
    if (v > best || (v == best && i < at)) { best = v; at = i; }
  }
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) {
    const float v = __shfl_xor(best, m, 64);
    const int i = __shfl_xor(at, m, 64);
    if (v > best || (v == best && i < at)) { best = v; at = i; }
  }
  if ((threadIdx.x & 63) == 0) { bv[threadIdx.x >> 6] = best; bi[threadIdx.x >> 6] = at; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 16; ++w)
      if (bv[w] > best || (bv[w] == best && bi[w] < at)) { best = bv[w]; at = bi[w]; }
    out[blockIdx.x] = at == 0x7fffffff ? 0 : at;
  }
}

}  // namespace lm

using namespace lm;

extern "C" int lm_residual_norm(float* x, int64_t ldx, const int* tokens, const void* embed, float embed_scale, const void* y,
                                int64_t ldy, const float* y_bias, const float* pair_w, int top, int pairs0, int shared, const float* post_w, const float* post_b,
                                const float* next_w, const float* next_b, void* h, int64_t ldh, const int* rows, int n_rows, int n,
                                int kind, int store_x, float eps, void* stream) {
  if (n_rows <= 0 || n <= 0 || n > ldx || ldx % 4 || (tokens && !embed) || (next_w && !h) || (h && (ldh % 4 || ldh < n)) || top < 0 ||
      (top > 0 && (!y || !pair_w)))
    return LM_EINVAL;
  ResidualArgs a{x, ldx, tokens, (const elem_t*)embed, embed_scale, (const elem_t*)y, ldy, y_bias, pair_w, top, pairs0, shared, post_w, post_b, next_w,
                 next_b, (elem_t*)h, ldh, rows, n, kind, store_x, eps};
  hipStream_t s = (hipStream_t)stream;
  const int64_t cols = ldx > ldh ? ldx : ldh;
#define LM_CASE(TH, NV) \
  if (cols <= 4 * TH * NV) { hipLaunchKernelGGL((residual_norm_kernel<TH, NV>), dim3(n_rows), dim3(TH), 0, s, a); return launch_status(); }
  LM_CASE(256, 1)
  if (n_rows <= 256) {      // latency: the whole workgroup on one piece of the row
    LM_CASE(512, 1) LM_CASE(1024, 1) LM_CASE(1024, 2) LM_CASE(1024, 4)
  }
  LM_CASE(256, 2) LM_CASE(256, 4) LM_CASE(256, 8) LM_CASE(256, 16)
#undef LM_CASE
  return LM_EINVAL;
}

extern "C" int lm_gated_rms(void* out, int64_t ldo, const void* o, int64_t ldi, const void* gate, int64_t ldg, const float* w,
                            int rows, int cols, int n, float eps, void* stream) {
  if (rows <= 0 || n <= 0 || n > cols || cols % 4 || ldo % 4 || ldi % 4 || ldg % 4) return LM_EINVAL;
  hipStream_t s = (hipStream_t)stream;
#define LM_CASE(NV)                                                                                                              \
  if (cols <= 1024 * NV) {                                                                                                       \
    hipLaunchKernelGGL((gated_rms_kernel<NV>), dim3(rows), dim3(ROW_THREADS), 0, s, (elem_t*)out, ldo, (const elem_t*)o, ldi,     \
                       (const elem_t*)gate, ldg, w, cols, n, eps);                                                               \
    return launch_status();                                                                                                      \
  }
  LM_CASE(1) LM_CASE(2) LM_CASE(4) LM_CASE(8) LM_CASE(16)
#undef LM_CASE
  return LM_EINVAL;
}

extern "C" int lm_gated_head_rms(void* out, int64_t ldo, const void* o, int64_t ldi, const void* gate, int64_t ldg, const float* w,
                                 int rows, int H, int dv, int n, float eps, int act, void* stream) {
  if (rows <= 0 || H <= 0 || (dv != 64 && dv != 128 && dv != 256) || n <= 0 || n > dv || ldo % 4 || ldi % 4 || ldg % 4 ||
      (act != LM_ACT_SILU && act != LM_ACT_SIGMOID))
    return LM_EINVAL;
  hipLaunchKernelGGL(gated_head_rms_kernel, dim3(rows), dim3(ROW_THREADS), 0, (hipStream_t)stream, (elem_t*)out, ldo, (const elem_t*)o,
                     ldi, (const elem_t*)gate, ldg, w, H * dv, dv, n, eps, act);
  return launch_status();
}

extern "C" int lm_glu(void* out, int64_t ldo, const void* x, int64_t ldx, const float* bias, int rows, int n, int act, void* stream) {
  if (rows <= 0 || n <= 0 || n % 16 || ldo % FR || ldx % FR || (act != LM_ACT_SILU && act != LM_ACT_GELU_TANH)) return LM_EINVAL;
  const dim3 grid((n + ROW_THREADS * FR - 1) / (ROW_THREADS * FR), (rows + GLU_ROWS - 1) / GLU_ROWS);
  hipLaunchKernelGGL(glu_kernel, grid, dim3(ROW_THREADS), 0, (hipStream_t)stream, (elem_t*)out, ldo, (const elem_t*)x, ldx, bias, rows, n,
                     act);
  return launch_status();
}

extern "C" int lm_rope_append(void* qkv, int64_t ld, const void* v_first, int64_t ldv, float lambda, const float* freq, int half,
                              const int* pos, const int* slot, void* kc, void* vc, int tokens, int H, int G, int dk, int dv,
                              void* stream) {
  if (tokens <= 0 || half < 0 || half > 256 || 2 * half > dk || G <= 0 || H % G || dk % FR || dv % FR || ld % FR || ldv % FR)
    return LM_EINVAL;
  RopeArgs a{(elem_t*)qkv, ld, (const elem_t*)v_first, ldv, lambda, freq, half, pos, slot, (elem_t*)kc, (elem_t*)vc, H, G, dk, dv};
  hipLaunchKernelGGL(rope_append_kernel, dim3(tokens), dim3(ROW_THREADS), 0, (hipStream_t)stream, a);
  return launch_status();
}

extern "C" int lm_argmax(int64_t* out, const float* z, int64_t ld, int rows, int n, void* stream) {
  if (rows <= 0 || n <= 0 || ld < n) return LM_EINVAL;
  hipLaunchKernelGGL(argmax_kernel, dim3(rows), dim3(1024), 0, (hipStream_t)stream, out, z, ld, n);
  return launch_status();
}

extern "C" int lm_abi_version(void) { return LM_ABI_VERSION; }
extern "C" int lm_elem_bytes(void) { return (int)sizeof(elem_t); }
