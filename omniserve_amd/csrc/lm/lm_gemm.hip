// Matrix products y = x W^T, one launch for a set of weight matrices ("groups"): a dense projection is one group, a mixture of
// experts is one group per expert over the tokens routed to it, plus one for the shared expert over all tokens.
//
//   lm_gemm_rows   few rows (decode): HBM bound.  A workgroup owns 16 or 32 channels of a group and streams their weights
//                  once; its waves split K and meet in LDS.  Weights are the A operand straight from global memory.
//   lm_gemm_tiles  many rows (prefill): MFMA bound.  128 x 128 tiles, both operands by LDS-DMA, double buffered.
//
// Epilogues: element type, f32 times a factor, or the gated unit silu(gate) * up of a matrix whose rows alternate in blocks of
// 16 between gate and up channels (both halves of a pair then sit in the same lane).
#include "lm_common.h"
#include "omniserve_lm.h"

namespace lm {

struct Part {        // a family of equally shaped groups
  const elem_t* w;   // [groups][n][k]
  const elem_t* x; int64_t ldx;
  void* y; int64_t ldy;
  int n, k;
};

struct GemmArgs {
  Part a, b;                  // a: groups 0 .. groups - 1 (rows by perm / off), b: one group over rows 0 .. rows_b - 1
  int groups;
  const int* perm;            // row of y for every sorted place (null: identity, rows_a rows)
  const int* off;             // [groups + 1] sorted places of each group
  int rows_a, rows_b;
  int x_div;                  // x row = y row / x_div (tokens of (token, choice) pairs)
  const int* tiles; const int* n_tiles;   // lm_gemm_tiles with perm: (group, first place) of every 128-row tile
  float scale;
};

template <int EPI>
__device__ __forceinline__ void store4(const Part& pt, int64_t row, int c, f32x4 v, f32x4 up, float scale) {
  if constexpr (EPI == LM_EPI_ELEM) {
    *(quad_t*)((elem_t*)pt.y + row * pt.ldy + c) = to_quad(v);
  } else if constexpr (EPI == LM_EPI_F32) {
    *(f32x4*)((float*)pt.y + row * pt.ldy + c) = v * scale;
  } else {
    f32x4 r;
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = silu(v[e]) * up[e];
    *(quad_t*)((elem_t*)pt.y + row * pt.ldy + c) = to_quad(r);
  }
}

// A workgroup owns 16 NR NW channels: NW groups of waves take NR 16-channel blocks each (they read the same rows of x, out of the
// CU's L1), the KW waves of a group split K and meet in LDS.  16 MB rows at a time; blockIdx.z takes every gridDim.z-th such part.
template <int NR, int MB, int NW, int KW, int EPI>
__global__ __launch_bounds__(64 * NW * KW) void gemm_rows_kernel(GemmArgs p) {
  constexpr int U = NR * MB >= 2 ? 4 : 8;       // k-steps requested together
  __shared__ __attribute__((aligned(16))) float red_all[NW][KW][16 * MB][16 * NR + 4];
  const int g = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int nw = wave / KW, kw = wave % KW, gt = tid - nw * 64 * KW;      // group, K part, thread within the group
  float(*red)[16 * MB][16 * NR + 4] = red_all[nw];
  const bool is_b = g >= p.groups;
  const Part& pt = is_b ? p.b : p.a;
  if ((int)blockIdx.x * 16 * NR * NW >= pt.n) return;
  const int n0 = (blockIdx.x * NW + nw) * 16 * NR;
  int first = 0, rows = is_b ? p.rows_b : p.rows_a;
  const int* perm = is_b ? nullptr : p.perm;
  if (perm) { first = p.off[g]; rows = p.off[g + 1] - first; }
  if (rows <= 0) return;
  const elem_t* w = pt.w + (is_b ? 0 : (int64_t)g * pt.n * pt.k);
  const int steps = pt.k / KSTEP, s0 = steps * kw / KW, s1 = steps * (kw + 1) / KW;
  const elem_t* wp[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int c = n0 + 16 * r + l15;
    wp[r] = w + (int64_t)(c < pt.n ? c : pt.n - 1) * pt.k + FR * l4;
  }
  const int div = is_b ? 1 : p.x_div;
  for (int m0 = 16 * MB * blockIdx.z; m0 < rows; m0 += 16 * MB * gridDim.z) {
    const elem_t* xp[MB];
#pragma unroll
    for (int m = 0; m < MB; ++m) {
      const int i = m0 + 16 * m + l15, ic = i < rows ? i : rows - 1;
      const int pair = perm ? perm[first + ic] : ic;
      xp[m] = pt.x + (int64_t)(pair / div) * pt.ldx + FR * l4;
    }
    const int mb = min(MB, (rows - m0 + 15) >> 4);     // row blocks with work (uniform)
    f32x4 acc[NR][MB];
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int m = 0; m < MB; ++m) acc[r][m] = zero4();
    frag_t wf[NR][U], wn[NR][U];
    auto request = [&](frag_t (&f)[NR][U], int s) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < NR; ++r) f[r][u] = __builtin_nontemporal_load((const frag_t*)(wp[r] + (int64_t)(s + u) * KSTEP));
    };
    auto multiply = [&](frag_t (&f)[NR][U], int s) {
#pragma unroll
      for (int m = 0; m < MB; ++m) {
        if (m < mb) {
          frag_t xf[U];
#pragma unroll
          for (int u = 0; u < U; ++u) xf[u] = *(const frag_t*)(xp[m] + (int64_t)(s + u) * KSTEP);
#pragma unroll
          for (int u = 0; u < U; ++u)
#pragma unroll
            for (int r = 0; r < NR; ++r) acc[r][m] = mma(f[r][u], xf[u], acc[r][m]);
        }
      }
    };
    int s = s0;
    if (s + U <= s1) request(wf, s);
    while (s + U <= s1) {              // the next U steps are on their way while these multiply
      if (s + 2 * U <= s1) request(wn, s + U);
      multiply(wf, s);
      s += U;
      if (s + U > s1) break;
      if (s + 2 * U <= s1) request(wf, s + U);
      multiply(wn, s);
      s += U;
    }
    for (; s < s1; ++s) {
      frag_t w1[NR];
#pragma unroll
      for (int r = 0; r < NR; ++r) w1[r] = *(const frag_t*)(wp[r] + (int64_t)s * KSTEP);
#pragma unroll
      for (int m = 0; m < MB; ++m) {
        if (m < mb) {
          const frag_t xf = *(const frag_t*)(xp[m] + (int64_t)s * KSTEP);
#pragma unroll
          for (int r = 0; r < NR; ++r) acc[r][m] = mma(w1[r], xf, acc[r][m]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int m = 0; m < MB; ++m) *(f32x4*)&red[kw][16 * m + l15][16 * r + 4 * l4] = acc[r][m];
    __syncthreads();
    constexpr int OB = EPI == LM_EPI_GLU ? NR / 2 : NR;      // 16-channel blocks of the result
    for (int i = gt; i < 16 * MB * OB * 4; i += 64 * KW) {
      const int m = i / (OB * 4), q = i - m * (OB * 4), blk = q >> 2, c4 = 4 * (q & 3);
      const int sb = EPI == LM_EPI_GLU ? 2 * blk : blk;
      if (m0 + m >= rows) continue;
      f32x4 v = zero4(), up = zero4();
#pragma unroll
      for (int k = 0; k < KW; ++k) {
        v += *(const f32x4*)&red[k][m][16 * sb + c4];
        if constexpr (EPI == LM_EPI_GLU) up += *(const f32x4*)&red[k][m][16 * sb + 16 + c4];
      }
      const int pair = perm ? perm[first + m0 + m] : m0 + m;
      const int c = (EPI == LM_EPI_GLU ? n0 / 2 : n0) + 16 * blk + c4;
      if (c < (EPI == LM_EPI_GLU ? pt.n / 2 : pt.n)) store4<EPI>(pt, pair, c, v, up, p.scale);
    }
    __syncthreads();
  }
}

constexpr int TM = 128, TN = 128, TROWB = 128, TK = TROWB / (int)sizeof(elem_t);     // rows, channels, k bytes / values per stage
typedef Tile<TROWB> KTile;

template <int EPI>
__global__ __launch_bounds__(256, 2) void gemm_tiles_kernel(GemmArgs p, int mt_a, int mt_b) {
  __shared__ __attribute__((aligned(16))) uint8_t wt0[TN * TROWB], wt1[TN * TROWB], xt0[TM * TROWB], xt1[TM * TROWB];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  // linear order: groups of 8 row tiles, all channel tiles of such a group before the next one; a contiguous range per XCD
  const int nt_a = (p.a.n + TN - 1) / TN, nt_b = mt_b ? (p.b.n + TN - 1) / TN : 0;
  const int mt = p.tiles ? p.n_tiles[0] : mt_a;              // row tiles of part a that exist
  int id = xcd_contiguous(blockIdx.x, mt_a * nt_a + mt_b * nt_b);
  if (id < 0) return;
  const bool is_b = id >= mt_a * nt_a;
  const Part& pt = is_b ? p.b : p.a;
  const int nt = is_b ? nt_b : nt_a, mts = is_b ? mt_b : mt_a;
  if (is_b) id -= mt_a * nt_a;
  constexpr int GM = 8;
  const int band = id / (GM * nt), in = id - band * GM * nt, bm = min(GM, mts - band * GM);
  const int mi = band * GM + in % bm, ni = in / bm;
  if (!is_b && mi >= mt) return;
  const int* perm = is_b ? nullptr : p.perm;
  int first, rows, g = 0;
  if (perm) {
    g = p.tiles[2 * mi];
    first = p.tiles[2 * mi + 1];
    rows = p.off[g + 1] - first;
  } else {
    first = mi * TM;
    rows = (is_b ? p.rows_b : p.rows_a) - first;
  }
  rows = min(rows, TM);
  const int n0 = ni * TN;
  const elem_t* w = pt.w + (int64_t)g * pt.n * pt.k;
  // DMA pieces of 8 rows: lane -> (row lane / 8, physical slot lane % 8); wave w carries pieces 4 w .. 4 w + 3 of both operands
  const elem_t *wsrc[4], *xsrc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 8 * (4 * wave + i) + (lane >> 3), s = (lane & 7) ^ KTile::swizzle(r);
    const int c = n0 + r < pt.n ? n0 + r : pt.n - 1;
    wsrc[i] = w + (int64_t)c * pt.k + s * FR;
    const int rr = r < rows ? r : rows - 1;
    const int xr = perm ? perm[first + rr] / p.x_div : first + rr;
    xsrc[i] = pt.x + (int64_t)xr * pt.ldx + s * FR;
  }
  auto stage = [&](uint8_t* wt, uint8_t* xt, int k0) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      dma16(wsrc[i] + k0, wt + 1024 * (4 * wave + i));
      dma16(xsrc[i] + k0, xt + 1024 * (4 * wave + i));
    }
  };
  const int wn = 64 * (wave & 1), wm = 64 * (wave >> 1);
  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = zero4();
  stage(wt0, xt0, 0);
  __syncthreads();
  auto step = [&](const uint8_t* wt, const uint8_t* xt, uint8_t* wnext, uint8_t* xnext, int knext) {
    frag_t a[2][4], b[2][4];
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a[s][i] = KTile::frag(wt, wn + 16 * i + l15, 4 * s + l4);
        b[s][i] = KTile::frag(xt, wm + 16 * i + l15, 4 * s + l4);
      }
    __builtin_amdgcn_sched_barrier(0);
    if (knext < pt.k) stage(wnext, xnext, knext);
    __builtin_amdgcn_sched_barrier(0);
    __builtin_amdgcn_s_setprio(1);
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mma(a[s][i], b[s][j], acc[i][j]);
    __builtin_amdgcn_s_setprio(0);
    __syncthreads();
  };
  for (int k0 = 0; k0 < pt.k; k0 += 2 * TK) {
    step(wt0, xt0, wt1, xt1, k0 + TK);
    if (k0 + TK < pt.k) step(wt1, xt1, wt0, xt0, k0 + 2 * TK);
  }
  if constexpr (EPI == LM_EPI_F32) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int m = wm + 16 * j + l15;
      if (m >= rows) continue;
      const int64_t row = perm ? perm[first + m] : first + m;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = n0 + wn + 16 * i + 4 * l4;
        if (c < pt.n) store4<EPI>(pt, row, c, acc[i][j], zero4(), p.scale);
      }
    }
  } else {
    // through LDS, so that a row leaves in whole 16-byte pieces of neighbouring lanes; a wave handles its own 64 rows x (64 or
    // 32) channels in two halves of 32 rows (all tiles have been read: the last step ended with a barrier)
    constexpr int OC = EPI == LM_EPI_GLU ? 32 : 64, PITCH = OC * (int)sizeof(elem_t) + 16, PPR = OC / FR;
    uint8_t* buf = wave == 0 ? wt0 : wave == 1 ? wt1 : wave == 2 ? xt0 : xt1;
    static_assert(32 * PITCH <= TN * TROWB, "a wave's half fits its buffer");
#pragma unroll
    for (int half = 0; half < 2; ++half) {
#pragma unroll
      for (int jj = 0; jj < 2; ++jj) {
        const int j = 2 * half + jj;
#pragma unroll
        for (int i = 0; i < 4; i += EPI == LM_EPI_GLU ? 2 : 1) {
          f32x4 v = acc[i][j];
          int c = 16 * i;
          if constexpr (EPI == LM_EPI_GLU) {
            c = 8 * i;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = silu(v[e]) * acc[i + 1][j][e];
          }
          *(quad_t*)(buf + (16 * jj + l15) * PITCH + (c + 4 * l4) * (int)sizeof(elem_t)) = to_quad(v);
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int i = 0; i < 32 * PPR / 64; ++i) {
        const int pc = 64 * i + lane, r = pc / PPR, q = pc % PPR;
        const int m = wm + 32 * half + r, c = (EPI == LM_EPI_GLU ? (n0 + wn) / 2 : n0 + wn) + q * FR;
        if (m < rows && c < (EPI == LM_EPI_GLU ? pt.n / 2 : pt.n)) {
          const int64_t row = perm ? perm[first + m] : first + m;
          *(frag_t*)((elem_t*)pt.y + row * pt.ldy + c) = *(const frag_t*)(buf + r * PITCH + q * 16);
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
    }
  }
}

static int check_part(const Part& p, int epi) {
  if (!p.w || !p.x || !p.y || p.n <= 0 || p.k <= 0 || p.k % 64 || p.n % 16 || p.ldx < p.k || p.ldx % FR || p.ldy % FR) return LM_EINVAL;
  if (epi == LM_EPI_GLU && p.n % 32) return LM_EINVAL;
  return LM_OK;
}

static int fill(GemmArgs& a, const LmGemmPart* pa, const LmGemmPart* pb, int groups, const int* perm, const int* off, int rows_a,
                int rows_b, int x_div, float scale, int epi) {
  auto conv = [](const LmGemmPart* s) {
    return Part{(const elem_t*)s->w, (const elem_t*)s->x, s->ldx, s->y, s->ldy, s->n, s->k};
  };
  if (!pa || groups <= 0 || x_div <= 0 || (groups > 1 && !perm) || (perm && !off) || epi < 0 || epi > LM_EPI_GLU) return LM_EINVAL;
  a.a = conv(pa);
  a.b = pb ? conv(pb) : Part{};
  if (check_part(a.a, epi) || (pb && check_part(a.b, epi))) return LM_EINVAL;
  a.groups = groups; a.perm = perm; a.off = off; a.rows_a = rows_a; a.rows_b = pb ? rows_b : 0; a.x_div = perm ? x_div : 1;
  a.tiles = nullptr; a.n_tiles = nullptr; a.scale = scale;
  return LM_OK;
}

template <int NR, int NW, int KW, int EPI>
static int launch_rows(const GemmArgs& a, int max_rows, int has_b, hipStream_t s) {
  const int n = has_b && a.b.n > a.a.n ? a.b.n : a.a.n;
  const int mb = max_rows <= 16 ? 1 : max_rows <= 32 ? 2 : 4;
  const dim3 grid((n + 16 * NR * NW - 1) / (16 * NR * NW), a.groups + has_b, a.perm ? 1 : (max_rows + 16 * mb - 1) / (16 * mb));
  const dim3 block(64 * NW * KW);
  if (mb == 1) hipLaunchKernelGGL((gemm_rows_kernel<NR, 1, NW, KW, EPI>), grid, block, 0, s, a);
  else if (mb == 2) hipLaunchKernelGGL((gemm_rows_kernel<NR, 2, NW, KW, EPI>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((gemm_rows_kernel<NR, 4, NW, KW, EPI>), grid, block, 0, s, a);
  return launch_status();
}

// Channels per workgroup: as many as still leave a workgroup for every CU (fewer reads of x).  A product of few channels over
// many rows (the router of a prompt) has its workgroups along the rows instead.
template <int EPI>
static int plan_rows(const GemmArgs& a, int max_rows, int has_b, hipStream_t s) {
  const int64_t n = (int64_t)a.groups * a.a.n;
  if constexpr (EPI == LM_EPI_GLU) {
    return launch_rows<2, 1, 8, EPI>(a, max_rows, has_b, s);
  } else {
    if (max_rows > 64) return launch_rows<2, 1, 8, EPI>(a, max_rows, has_b, s);
    if (n >= 128 * 256) return launch_rows<2, 4, 2, EPI>(a, max_rows, has_b, s);
    if (n >= 64 * 240) return launch_rows<1, 4, 2, EPI>(a, max_rows, has_b, s);
    if (n >= 32 * 240) return launch_rows<1, 2, 4, EPI>(a, max_rows, has_b, s);
    return launch_rows<1, 1, 8, EPI>(a, max_rows, has_b, s);
  }
}

}  // namespace lm

using namespace lm;

extern "C" int lm_gemm_rows(const LmGemmPart* pa, const LmGemmPart* pb, int groups, const int* perm, const int* off, int rows_a,
                            int rows_b, int x_div, int max_rows, float scale, int epi, void* stream) {
  GemmArgs a;
  if (fill(a, pa, pb, groups, perm, off, rows_a, rows_b, x_div, scale, epi) || max_rows <= 0) return LM_EINVAL;
  hipStream_t s = (hipStream_t)stream;
  const int has_b = pb && rows_b > 0;
  if (epi == LM_EPI_GLU) return plan_rows<LM_EPI_GLU>(a, max_rows, has_b, s);
  return epi == LM_EPI_F32 ? plan_rows<LM_EPI_F32>(a, max_rows, has_b, s) : plan_rows<LM_EPI_ELEM>(a, max_rows, has_b, s);
}

extern "C" int lm_gemm_tiles(const LmGemmPart* pa, const LmGemmPart* pb, int groups, const int* perm, const int* off,
                             const int* tiles, const int* n_tiles, int max_tiles, int rows_a, int rows_b, int x_div,
                             float scale, int epi, void* stream) {
  GemmArgs a;
  if (fill(a, pa, pb, groups, perm, off, rows_a, rows_b, x_div, scale, epi)) return LM_EINVAL;
  if (perm && (!tiles || !n_tiles || max_tiles <= 0)) return LM_EINVAL;
  a.tiles = perm ? tiles : nullptr;
  a.n_tiles = n_tiles;
  const int mt_a = perm ? max_tiles : (rows_a + TM - 1) / TM, mt_b = pb && rows_b > 0 ? (rows_b + TM - 1) / TM : 0;
  const int64_t total = (int64_t)mt_a * ((a.a.n + TN - 1) / TN) + (int64_t)mt_b * (mt_b ? (a.b.n + TN - 1) / TN : 0);
  if (total <= 0 || total > (1 << 30)) return LM_EINVAL;
  const dim3 grid((unsigned)(8 * ((total + 7) / 8)));
  hipStream_t s = (hipStream_t)stream;
  if (epi == LM_EPI_ELEM) hipLaunchKernelGGL((gemm_tiles_kernel<LM_EPI_ELEM>), grid, dim3(256), 0, s, a, mt_a, mt_b);
  else if (epi == LM_EPI_F32) hipLaunchKernelGGL((gemm_tiles_kernel<LM_EPI_F32>), grid, dim3(256), 0, s, a, mt_a, mt_b);
  else hipLaunchKernelGGL((gemm_tiles_kernel<LM_EPI_GLU>), grid, dim3(256), 0, s, a, mt_a, mt_b);
  return launch_status();
}
