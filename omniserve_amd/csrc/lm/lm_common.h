// Shared device helpers of the engine's layer kernels (gfx950, wave64).  The library is compiled once per element type:
// LM_ELEM = 0 bf16, 1 f32.  Every matrix product goes through 16x16 MFMA tiles with f32 accumulators; the two element types
// differ only in how many k values a 16-byte operand fragment holds, so one kernel source serves both:
//
//   fragment (16 bytes per lane)  lane l15 = row (A) / column (B), l4 = lane / 16 picks the k group:
//                                 bf16: k = 32 s + 8 l4 + (0..7), one 16x16x32 MFMA; f32: k = 16 s + 4 l4 + (0..3), four
//                                 16x16x4 MFMAs (both operands permute k alike)
//   quad (4 k values per lane)    k = 16 t + 4 l4 + (0..3): what one MFMA's accumulator holds per lane, so a result tile can
//                                 be the operand of the next product without leaving registers
//   accumulator                   column l15, rows 4 l4 + (0..3)
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#ifndef LM_ELEM
#error "LM_ELEM must be 0 (bf16) or 1 (f32)"
#endif

#define LM_OK 0
#define LM_EINVAL (-22)
#define LM_ELAUNCH (-5)

namespace lm {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x2 __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef int i32x4 __attribute__((ext_vector_type(4)));

#if LM_ELEM == 0
typedef __bf16 elem_t;
typedef bf16x8 frag_t;
typedef bf16x4 quad_t;
constexpr bool SPLIT = true;     // f32 factors enter a matrix product as the sum of two bf16 operands
#else
typedef float elem_t;
typedef f32x4 frag_t;
typedef f32x4 quad_t;
constexpr bool SPLIT = false;
#endif
constexpr int FR = 16 / (int)sizeof(elem_t);     // elements per fragment
constexpr int KSTEP = 4 * FR;                    // k values per fragment product
constexpr int NOPND = SPLIT ? 2 : 1;             // operands an f32 factor needs
constexpr int PAGE = 64;                         // tokens per cache page

__device__ __forceinline__ f32x4 zero4() { return (f32x4){0.f, 0.f, 0.f, 0.f}; }

__device__ __forceinline__ f32x4 mma(frag_t a, frag_t b, f32x4 c) {
#if LM_ELEM == 0
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
#else
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
#endif
}

// k = two neighbouring 16-blocks, one quad each
__device__ __forceinline__ f32x4 mma_quads(quad_t a0, quad_t a1, quad_t b0, quad_t b1, f32x4 c) {
#if LM_ELEM == 0
  return mma(__builtin_shufflevector(a0, a1, 0, 1, 2, 3, 4, 5, 6, 7), __builtin_shufflevector(b0, b1, 0, 1, 2, 3, 4, 5, 6, 7), c);
#else
  return mma(a1, b1, mma(a0, b0, c));
#endif
}

__device__ __forceinline__ quad_t to_quad(f32x4 x) {
#if LM_ELEM == 0
  return (quad_t){(elem_t)x[0], (elem_t)x[1], (elem_t)x[2], (elem_t)x[3]};
#else
  return x;
#endif
}
__device__ __forceinline__ f32x4 from_quad(quad_t q) { return (f32x4){(float)q[0], (float)q[1], (float)q[2], (float)q[3]}; }

// x = q[0] + q[1] to 16 significand bits (bf16), q[0] = x (f32)
__device__ __forceinline__ void split_quad(f32x4 x, quad_t (&q)[NOPND]) {
  q[0] = to_quad(x);
  if constexpr (SPLIT) q[NOPND - 1] = to_quad(x - from_quad(q[0]));
}

__device__ __forceinline__ float sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }      // (rcp: within an ulp)
__device__ __forceinline__ float silu(float z) { return z * sigmoid(z); }
__device__ __forceinline__ float gelu_tanh(float z) {      // 0.5 z (1 + tanh u) = z sigmoid(2 u)
  return z * sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z));
}
// log(1 + e^z)
__device__ __forceinline__ float softplus(float z) {
  const float e = __expf(-fabsf(z)), u = 1.0f + e, d = u - 1.0f;
  return fmaxf(z, 0.f) + (d == 0.f ? e : __logf(u) * e * __builtin_amdgcn_rcpf(d));      // log1p(e) without the cancellation
}
constexpr float LOG2E = 1.4426950408889634f;

// lam^n for n >= 0, from log2(lam)
__device__ __forceinline__ float power(float log2_lam, int n) { return n == 0 ? 1.0f : __builtin_amdgcn_exp2f((float)n * log2_lam); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) v += __shfl_xor(v, m, 64);
  return v;
}

// the four lanes that share l15
__device__ __forceinline__ float column_max(float v) {
  v = fmaxf(v, __shfl_xor(v, 16, 64));
  return fmaxf(v, __shfl_xor(v, 32, 64));
}
__device__ __forceinline__ float column_sum(float v) {
  v += __shfl_xor(v, 16, 64);
  return v + __shfl_xor(v, 32, 64);
}

// LDS tile of rows of ROWB bytes in 16-byte slots, slot s of row r stored at s ^ swizzle(r).  A fragment read (ds_read_b128)
// serves lanes {0-3, 12-15, 20-23, 24-27} and the like together, i.e. rows 0-3 and 12-15 at one slot with rows 4-11 at its
// neighbour: the swizzles of rows 4-11 are closed under flipping the low bit, so 16 different places of a 256-byte line answer.
// A transposed read serves 8 consecutive rows at one 32-byte block: their swizzles differ above the low bit.
template <int ROWB>
struct Tile {
  static constexpr int NS = ROWB / 16;
  static_assert(NS >= 8 && NS % 8 == 0, "row size");
  // The same accesses from per-lane byte offsets, for rows of a power of two bytes: what depends on the block is one XOR.  A loop
  // that keeps the three offsets from the optimiser (Offsets::forget) does not hold an address register per block.
  struct Offsets {
    int frag, quad, col;
    __device__ __forceinline__ Offsets(int l15, int l4) {
      static_assert((NS & (NS - 1)) == 0, "row size");
      const int row = l15 * ROWB, r = 4 * l4 + (l15 >> 2);
      frag = row + ((l4 ^ swizzle(l15)) << 4);
      quad = sizeof(elem_t) == 2 ? row + (((l4 >> 1) ^ swizzle(l15)) << 4) + 8 * (l4 & 1) : frag;
      col = r * ROWB + ((((l15 & 3) >> 1) ^ swizzle(r)) << 4) + 8 * (l15 & 1);
    }
    __device__ __forceinline__ void forget() { asm volatile("" : "+v"(frag), "+v"(quad), "+v"(col)); }
  };
  __device__ __forceinline__ static frag_t frag(const uint8_t* t, const Offsets& o, int row0, int k) {      // row row0 + l15, step k
    return *(const frag_t*)(t + row0 * ROWB + (o.frag ^ (k << 6)));
  }
  __device__ __forceinline__ static quad_t quad(const uint8_t* t, const Offsets& o, int row0, int blk) {
    return *(const quad_t*)(t + row0 * ROWB + (o.quad ^ (blk * 16 * (int)sizeof(elem_t))));
  }
  __device__ __forceinline__ static quad_t column_quad(const uint8_t* t, const Offsets& o, int row0, int cblk, int l15, int l4) {
#if LM_ELEM == 0
    return transposed(t + row0 * ROWB + (o.col ^ (cblk << 5)));
#else
    return column_quad(t, row0, cblk, l15, l4);
#endif
  }
  __device__ __forceinline__ static int swizzle(int row) {
    if constexpr (NS / 8 % 2 == 1) { // an odd number of half lines: neighbouring rows start in different halves
      const int q = (row >> 1) & 7;
      return (((q ^ ((q >> 1) & 2)) & 3) << 1) | (q >> 2);
    }
    const int r = row & 15;
    return (((r ^ ((r >> 1) & 4)) & 7) << 1) | (r >> 3);
  }
  __device__ __forceinline__ static int slot(int row, int s) { return row * ROWB + ((s ^ swizzle(row)) << 4); }
  // element col of row, byte offset
  __device__ __forceinline__ static int at(int row, int col) {
    const int b = col * (int)sizeof(elem_t);
    return slot(row, b >> 4) + (b & 15);
  }
  __device__ __forceinline__ static frag_t frag(const uint8_t* t, int row, int s) { return *(const frag_t*)(t + slot(row, s)); }
  // row, k = 16 blk + 4 l4 + (0..3)
  __device__ __forceinline__ static quad_t quad(const uint8_t* t, int row, int blk, int l4) {
    return *(const quad_t*)(t + at(row, 16 * blk + 4 * l4));
  }
#if LM_ELEM == 0
  __device__ __forceinline__ static quad_t transposed(const uint8_t* p) {
    typedef __bf16 tr4 __attribute__((__vector_size__(4 * sizeof(__bf16))));
    const tr4 r = __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
        (__attribute__((address_space(3))) tr4*)(__attribute__((address_space(3))) void*)(p));
    return (quad_t){r[0], r[1], r[2], r[3]};
  }
#endif
  // column 16 cblk + l15 of rows row0 + 4 l4 + (0..3)
  __device__ __forceinline__ static quad_t column_quad(const uint8_t* t, int row0, int cblk, int l15, int l4) {
#if LM_ELEM == 0
    // lane L of a 16-lane group passes the address of elements 4 (L & 3) .. + 3 of row L >> 2 and receives column L
    return transposed(t + at(row0 + 4 * l4 + (l15 >> 2), 16 * cblk + 4 * (l15 & 3)));
#else
    quad_t q;
#pragma unroll
    for (int i = 0; i < 4; ++i) q[i] = *(const float*)(t + at(row0 + 4 * l4 + i, 16 * cblk + l15));
    return q;
#endif
  }
};

// 16 bytes per lane, global -> LDS; the destination is lane-linear from a wave-uniform base
__device__ __forceinline__ void dma16(const void* src, void* lds_wave_base) {
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                   (__attribute__((address_space(3))) void*)lds_wave_base, 16, 0, 0);
}

// The same hidden from the compiler, which would wait for every DMA in flight in front of the next LDS read.  The kernel counts the
// pieces itself (wait_pieces).  M0 is the compiler's: saved and restored.
__device__ __forceinline__ void dma16_uncounted(const void* src, uint32_t lds_dst) {
  uint32_t keep;
  lds_dst = __builtin_amdgcn_readfirstlane(lds_dst);      // (uniform already; says so where the compiler cannot see it)
  asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
               : "=&s"(keep)
               : "v"(src), "s"(lds_dst)
               : "memory");
}
template <int N>
__device__ __forceinline__ void wait_pieces() {
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory");
}

// Workgroups are dealt round-robin to the 8 XCDs: hands every XCD one contiguous range of [0, total).  The grid has
// 8 * ceil(total / 8) workgroups; returns -1 for the surplus.
__device__ __forceinline__ int xcd_contiguous(int wid, int total) {
  const int per = (total + 7) >> 3, id = (wid & 7) * per + (wid >> 3);
  return id < total ? id : -1;
}

template <typename K>
static inline int allow_lds(K kernel, size_t bytes) {
  if (bytes <= 65536) return LM_OK;
  return hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) == hipSuccess ? LM_OK
                                                                                                                  : LM_EINVAL;
}
static inline int launch_status() { return hipGetLastError() == hipSuccess ? LM_OK : LM_ELAUNCH; }

}  // namespace lm
