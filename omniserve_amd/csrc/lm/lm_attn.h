// What the prefill and the decode attention share: the online softmax over the keys a lane holds.
//
// Scores are formed transposed (S^T = K q^T): a lane then holds 4 keys of one query per 16-key block, which is exactly the
// quad layout of the second product O^T = V^T P^T -- probabilities never leave the registers.  They are f32; for the bf16
// matrix product each one is the sum of two bf16 operands (split_quad).
#pragma once
#include "lm_common.h"

namespace lm {

constexpr float NEG = -1e30f;      // a masked score, and the running maximum before the first key

// x: raw scores, masked ones NEG; scale > 0 includes log2(e).  Updates the running maximum and the lane's part of the running
// sum, leaves the probabilities as operands; returns the factor of everything accumulated so far.
template <int NBLK>
__device__ __forceinline__ float softmax_step(const f32x4 (&x)[NBLK], float scale, float& m_run, float& l_run,
                                              quad_t (&pq)[NBLK][NOPND]) {
  float t = NEG;
#pragma unroll
  for (int u = 0; u < NBLK; ++u)
#pragma unroll
    for (int r = 0; r < 4; ++r) t = fmaxf(t, x[u][r]);
  t = column_max(t);
  const float m_new = t <= NEG ? m_run : fmaxf(m_run, t * scale);
  const float m_sub = m_new <= NEG ? 0.f : m_new;            // no key seen yet: every probability underflows to 0
  const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
  float sum = 0.f;
#pragma unroll
  for (int u = 0; u < NBLK; ++u) {
    f32x4 e;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      e[r] = __builtin_amdgcn_exp2f(__builtin_fmaf(x[u][r], scale, -m_sub));
      sum += e[r];
    }
    split_quad(e, pq[u]);
  }
  l_run = l_run * alpha + sum;
  m_run = m_new;
  return alpha;
}

// Parts [B][H][nsplit][2 + dv] (maximum, sum, weighted values) of decode attention -> [B][H][dv].  One workgroup per (sequence,
// head); at most 64 parts: lane s of every wave holds the maximum and sum of part s.
static __global__ __launch_bounds__(256) void attn_merge_kernel(const float* part, int nsplit, const int* pos, const elem_t* gate,
                                                                int64_t ldg, elem_t* o, int64_t ldo, int H, int dv) {
  const int b = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63;
  if (pos[b] < 0) return;
  const float* q = part + ((int64_t)b * H + h) * nsplit * (dv + 2);
  const int64_t step = dv + 2;
  const bool in = lane < nsplit;
  const float ms = in ? q[lane * step] : NEG, ls = in ? q[lane * step + 1] : 0.f;
  float m = ms;
#pragma unroll
  for (int k = 32; k > 0; k >>= 1) m = fmaxf(m, __shfl_xor(m, k, 64));
  const float f = __builtin_amdgcn_exp2f(ms - m), inv = 1.0f / wave_sum(f * ls);
  for (int d0 = 0; d0 < dv; d0 += 256) {
    const int d = d0 + threadIdx.x;
    float y = 0.f;
    for (int s0 = 0; s0 < nsplit; s0 += 8) {
      float v[8];
#pragma unroll
      for (int s = 0; s < 8; ++s) v[s] = d < dv && s0 + s < nsplit ? q[(s0 + s) * step + 2 + d] : 0.f;
#pragma unroll
      for (int s = 0; s < 8; ++s) y += __shfl(f, s0 + s, 64) * v[s];
    }
    if (d >= dv) continue;
    y *= inv;
    if (gate) y *= sigmoid((float)gate[(int64_t)b * ldg + (int64_t)h * dv + d]);
    o[(int64_t)b * ldo + (int64_t)h * dv + d] = (elem_t)y;
  }
}

}  // namespace lm
