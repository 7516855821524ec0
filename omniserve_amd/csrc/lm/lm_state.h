// What the single-token kernels of the recurrent layers share: one workgroup owns one head's state [dk][dv] (f32), thread =
// 4 value columns x dk / 16 rows, all of them in registers; sums over the rows meet in LDS.
#pragma once
#include "lm_common.h"

namespace lm {

constexpr int STATE_GROUPS = 16;                 // row groups

struct HeadOut {                                 // RMS norm over n of dv columns, times w, times silu(gate)
  const elem_t* gate;                            // of this head
  const float* w;
  int n;
  float eps;
};

// acc: this thread's part of sum_rows q S; the first wave returns with the sums of its 4 columns (lane < dv / 4)
template <int DV>
__device__ __forceinline__ f32x4 over_groups(f32x4 acc, f32x4 (*red)[DV / 4], int grp, int col) {
  red[grp][col] = acc;
  __syncthreads();
  f32x4 y = red[0][col];
#pragma unroll
  for (int g = 1; g < STATE_GROUPS; ++g) y += red[g][col];
  return y;
}

template <int DV>
__device__ __forceinline__ void head_out(f32x4 y, const HeadOut& p, elem_t* o) {      // threads 0 .. DV / 4 - 1, one wave
  const int col = threadIdx.x;
  float ss = (y[0] * y[0] + y[1] * y[1]) + (y[2] * y[2] + y[3] * y[3]);
#pragma unroll
  for (int m = DV / 8; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
  const float r = 1.0f / sqrtf(ss / (float)p.n + p.eps);
  const f32x4 g = from_quad(*(const quad_t*)(p.gate + 4 * col)), w = *(const f32x4*)(p.w + 4 * col);
#pragma unroll
  for (int e = 0; e < 4; ++e) y[e] *= r * w[e] * silu(g[e]);
  *(quad_t*)(o + 4 * col) = to_quad(y);
}

}  // namespace lm
