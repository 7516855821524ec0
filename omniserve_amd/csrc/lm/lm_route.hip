// Expert choice and the order of the grouped products: per token the `top` largest router logits (ties: the lower expert) and
// their softmax; then the (token, choice) pairs sorted by expert -- off[experts + 1], perm[pairs] -- and the row tiles of
// every expert for lm_gemm_tiles.
#include "lm_common.h"
#include "omniserve_lm.h"

namespace lm {

constexpr int MAX_EXPERTS = 512, MAX_TOP = 16;
constexpr int CHOOSE_TOKENS = 16;      // tokens per workgroup of route_choose_kernel

// one wave per token; lane l holds its EPL experts l, l + 64, ... and counts for each how many come before it in the order
// (larger logit, then lower number): the first `top` are the choice
template <int EPL>
__device__ __forceinline__ void choose(const float* z, const float* bias, int experts, int top, int lane, int* ids, float* wts) {
  float v[EPL];
  int before[EPL];
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    const int e = lane + 64 * i;
    const float x = e < experts ? z[e] + (bias ? bias[e] : 0.f) : -INFINITY;
    v[i] = x == x ? x : -INFINITY;        // (NaN: last)
    before[i] = 0;
  }
#pragma unroll
  for (int b = 0; b < EPL; ++b) {
    const int n = min(64, experts - 64 * b);
    for (int l = 0; l < n; ++l) {
      const float o = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v[b]), l));
      const int oe = 64 * b + l;
#pragma unroll
      for (int i = 0; i < EPL; ++i) before[i] += (int)(o > v[i]) | ((int)(o == v[i]) & (int)(oe < lane + 64 * i));
    }
  }
  float best = v[0];
#pragma unroll
  for (int i = 1; i < EPL; ++i) best = fmaxf(best, v[i]);
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) best = fmaxf(best, __shfl_xor(best, m, 64));
  if (best == -INFINITY) best = 0.f;
  float ex[EPL], sum = 0.f;
#pragma unroll
  for (int i = 0; i < EPL; ++i) {
    ex[i] = before[i] < top ? __expf(v[i] - best) : 0.f;
    sum += ex[i];
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int i = 0; i < EPL; ++i)
    if (before[i] < top && lane + 64 * i < experts) {
      ids[before[i]] = lane + 64 * i;
      wts[before[i]] = ex[i] / sum;
    }
}

// everything for up to 64 tokens in one workgroup
template <int EPL>
__global__ __launch_bounds__(1024) void route_small_kernel(const float* z, int64_t ldz, const float* bias, int tokens, int experts,
                                                           int top, float* wts, int* off, int* perm) {
  __shared__ int ids[64 * MAX_TOP], count[MAX_EXPERTS], start[MAX_EXPERTS + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, pairs = tokens * top;
  for (int e = tid; e < experts; e += 1024) count[e] = 0;
  for (int t = wave; t < tokens; t += 16) choose<EPL>(z + (int64_t)t * ldz, bias, experts, top, lane, ids + t * top, wts + (int64_t)t * top);
  __syncthreads();
  int rank = 0, e = 0;
  if (tid < pairs) {
    e = ids[tid];
    rank = atomicAdd(&count[e], 1);
  }
  __syncthreads();
  if (wave == 0) {                   // prefix sum of the counts, 64 experts at a time
    int base = 0;
    for (int e0 = 0; e0 < experts; e0 += 64) {
      const int c = e0 + lane < experts ? count[e0 + lane] : 0;
      int s = c;
#pragma unroll
      for (int m = 1; m < 64; m <<= 1) {
        const int o = __shfl_up(s, m, 64);
        if (lane >= m) s += o;
      }
      if (e0 + lane < experts) start[e0 + lane] = base + s - c;
      base += __shfl(s, 63, 64);
    }
    if (lane == 0) start[experts] = base;
  }
  __syncthreads();
  if (tid < pairs) perm[start[e] + rank] = tid;
  for (int i = tid; i <= experts; i += 1024) off[i] = start[i];
}

// many tokens: choices with their rank inside the expert (counts aggregated per workgroup before the global atomics) ...
template <int EPL>
__global__ __launch_bounds__(256) void route_choose_kernel(const float* z, int64_t ldz, const float* bias, int tokens, int experts,
                                                           int top, float* wts, int* ids, int* rank, int* count) {
  __shared__ int hist[MAX_EXPERTS], base[MAX_EXPERTS], lid[CHOOSE_TOKENS * MAX_TOP];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, t0 = blockIdx.x * CHOOSE_TOKENS, n = min(CHOOSE_TOKENS, tokens - t0);
  for (int e = tid; e < experts; e += 256) hist[e] = 0;
  for (int t = wave; t < n; t += 4)
    choose<EPL>(z + (int64_t)(t0 + t) * ldz, bias, experts, top, lane, lid + t * top, wts + (int64_t)(t0 + t) * top);
  __syncthreads();
  int r[CHOOSE_TOKENS * MAX_TOP / 256];
#pragma unroll
  for (int i = 0; i < CHOOSE_TOKENS * MAX_TOP / 256; ++i)
    if (tid + 256 * i < n * top) r[i] = atomicAdd(&hist[lid[tid + 256 * i]], 1);
  __syncthreads();
  for (int e = tid; e < experts; e += 256) base[e] = hist[e] ? atomicAdd(&count[e], hist[e]) : 0;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < CHOOSE_TOKENS * MAX_TOP / 256; ++i) {
    const int k = tid + 256 * i;
    if (k < n * top) {
      ids[(int64_t)t0 * top + k] = lid[k];
      rank[(int64_t)t0 * top + k] = base[lid[k]] + r[i];
    }
  }
}

// ... offsets and row tiles (entries past the last tile: no rows) ...
__global__ __launch_bounds__(512) void route_offsets_kernel(const int* count, int experts, int max_tiles, int* off, int* tiles) {
  __shared__ int s_off[MAX_EXPERTS], s_tile[MAX_EXPERTS];
  const int e = threadIdx.x, c = e < experts ? count[e] : 0, nt = (c + LM_TILE_ROWS - 1) / LM_TILE_ROWS;
  s_off[e] = c;
  s_tile[e] = nt;
  __syncthreads();
  for (int m = 1; m < 512; m <<= 1) {
    const int a = e >= m ? s_off[e - m] : 0, b = e >= m ? s_tile[e - m] : 0;
    __syncthreads();
    s_off[e] += a;
    s_tile[e] += b;
    __syncthreads();
  }
  i32x4* out = (i32x4*)tiles;
  if (e < experts) {
    const int o = s_off[e] - c, t = s_tile[e] - nt;
    off[e] = o;
    for (int i = 0; i < nt; ++i) out[t + i] = (i32x4){e, o + LM_TILE_ROWS * i, min(LM_TILE_ROWS, c - LM_TILE_ROWS * i), 0};
    if (e == experts - 1) off[experts] = s_off[e];
  }
  for (int t = s_tile[511] + e; t < max_tiles; t += 512) out[t] = (i32x4){0, 0, 0, 0};
}

// ... and the pairs in their places
__global__ __launch_bounds__(256) void route_scatter_kernel(const int* ids, const int* rank, const int* off, int pairs, int* perm) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < pairs) perm[off[ids[i]] + rank[i]] = i;
}

__global__ __launch_bounds__(512) void clear_kernel(int* p, int n) {
  if ((int)threadIdx.x < n) p[threadIdx.x] = 0;
}

}  // namespace lm

using namespace lm;

// scratch_i32: lm_route_scratch_words(tokens, experts, top) words (more than 64 tokens only)
extern "C" int64_t lm_route_scratch_words(int tokens, int experts, int top) { return MAX_EXPERTS + 2 * (int64_t)tokens * top; }
extern "C" int lm_route_max_tiles(int tokens, int experts, int top) {
  const int64_t pairs = (int64_t)tokens * top;
  return (int)(pairs / LM_TILE_ROWS + (pairs < experts ? pairs : experts));
}

extern "C" int lm_route(const float* z, int64_t ldz, const float* bias, int tokens, int experts, int top, float* wts, int* off,
                        int* perm, int* tiles, int* scratch_i32, void* stream) {
  if (tokens <= 0 || experts <= 0 || experts > MAX_EXPERTS || top <= 0 || top > MAX_TOP || top > experts || ldz < experts ||
      (int64_t)tokens * top > (1 << 28))
    return LM_EINVAL;
  hipStream_t s = (hipStream_t)stream;
  if (tokens <= 64 && !tiles) {
    auto k = experts <= 64 ? route_small_kernel<1> : experts <= 128 ? route_small_kernel<2> : route_small_kernel<MAX_EXPERTS / 64>;
    hipLaunchKernelGGL(k, dim3(1), dim3(1024), 0, s, z, ldz, bias, tokens, experts, top, wts, off, perm);
    return launch_status();
  }
  if (!tiles || !scratch_i32) return LM_EINVAL;
  const int pairs = tokens * top;
  int *count = scratch_i32, *ids = count + MAX_EXPERTS, *rank = ids + pairs;
  hipLaunchKernelGGL(clear_kernel, dim3(1), dim3(512), 0, s, count, MAX_EXPERTS);
  auto k = experts <= 64 ? route_choose_kernel<1> : experts <= 128 ? route_choose_kernel<2> : route_choose_kernel<MAX_EXPERTS / 64>;
  hipLaunchKernelGGL(k, dim3((tokens + CHOOSE_TOKENS - 1) / CHOOSE_TOKENS), dim3(256), 0, s, z, ldz, bias, tokens, experts, top, wts, ids, rank, count);
  hipLaunchKernelGGL(route_offsets_kernel, dim3(1), dim3(512), 0, s, count, experts,
                     lm_route_max_tiles(tokens, experts, top), off, tiles);
  hipLaunchKernelGGL(route_scatter_kernel, dim3((pairs + 255) / 256), dim3(256), 0, s, ids, rank, off, pairs, perm);
  return launch_status();
}
