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

}  // namespace lm
