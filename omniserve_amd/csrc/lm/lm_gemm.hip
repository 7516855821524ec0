// Matrix products y = x W^T, one launch for a set of weight matrices ("groups"): a dense projection is one group, a mixture of
// experts is one group per expert over the tokens routed to it, plus one for the shared expert over all tokens.
//
//   lm_gemm_rows   few rows (decode): HBM bound.  A workgroup owns 16 or 32 channels of a group and streams their weights
//                  once; its waves split K and meet in LDS.  Weights are the A operand straight from global memory.
//   lm_gemm_tiles  many rows (prefill): MFMA bound.  256 x 128 tiles, both operands by LDS-DMA, two stages ahead.
//
// Epilogues: element type, f32 times a factor, the gated unit act(gate + bias) * (up + bias) of a matrix whose rows alternate in
// blocks of 16 between gate and up channels (both halves of a pair then sit in the same lane), or the product with sigmoid(gate).
#include "lm_common.h"
#include "omniserve_lm.h"

namespace lm {

struct Part {        // a family of equally shaped groups
  const elem_t* w;   // [groups][n][k]
  const elem_t* x; int64_t ldx;
  void* y; int64_t ldy;
  int n, k;
  int64_t gx, gy;            // without perm: columns of x / y between neighbouring groups
  const float* bias;         // [n] added to the products of a gated unit (or null)
  const elem_t* gate;        // LM_EPI_GATE: the factor's argument, laid out like y
  int64_t ldg;
};

struct GemmArgs {
  Part a, b;                  // a: groups 0 .. groups - 1 (rows by perm / off), b: one group over rows 0 .. rows_b - 1
  int groups;
  const int* perm;            // row of y for every sorted place (null: identity, rows_a rows)
  const int* off;             // [groups + 1] sorted places of each group
  int rows_a, rows_b;
  int x_div;                  // x row = y row / x_div (tokens of (token, choice) pairs)
  const int* tiles;           // lm_gemm_tiles with perm: (group, first place, rows, 0) of every row tile, rows 0: none
  float scale;
  int act;                    // of the gated unit
};

__device__ __forceinline__ f32x4 glu(const Part& pt, int act, int c, f32x4 gate, f32x4 up) {      // c: gate channel's row in w, a multiple of 4
  if (pt.bias) {
    gate += *(const f32x4*)(pt.bias + c);
    up += *(const f32x4*)(pt.bias + c + 16);
  }
  f32x4 r;
  if (act == LM_ACT_GELU_TANH) {
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = gelu_tanh(gate[e]) * up[e];
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = silu(gate[e]) * up[e];
  }
  return r;
}

template <int EPI>
__device__ __forceinline__ void store4(const Part& pt, int64_t row, int c, int64_t y0, f32x4 v, float scale) {
  if constexpr (EPI == LM_EPI_ELEM || EPI == LM_EPI_GLU) {
    *(quad_t*)((elem_t*)pt.y + row * pt.ldy + y0 + c) = to_quad(v);
  } else if constexpr (EPI == LM_EPI_F32) {
    *(f32x4*)((float*)pt.y + row * pt.ldy + y0 + c) = v * scale;
  } else {
    const f32x4 z = from_quad(*(const quad_t*)(pt.gate + row * pt.ldg + y0 + c));
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= sigmoid(z[e]);
    *(quad_t*)((elem_t*)pt.y + row * pt.ldy + y0 + c) = to_quad(v);
  }
}

// A workgroup owns NR 16-channel blocks; its KW waves split K and meet in LDS.  16 MB rows at a time; blockIdx.z takes every
// gridDim.z-th such part.
template <int NR, int MB, int KW, int EPI>
__global__ __launch_bounds__(64 * KW) void gemm_rows_kernel(GemmArgs p) {
  constexpr int U = NR > 1 ? 4 : 8;             // k-steps of weights requested together (a multiple of 4: see xf)
  __shared__ __attribute__((aligned(16))) float red[KW][16 * MB][16 * NR + 4];
  const int g = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const bool is_b = g >= p.groups;
  const Part& pt = is_b ? p.b : p.a;
  const int n0 = blockIdx.x * 16 * NR;
  if (n0 >= pt.n) return;
  int first = 0, rows = is_b ? p.rows_b : p.rows_a;
  const int* perm = is_b ? nullptr : p.perm;
  if (perm) { first = p.off[g]; rows = p.off[g + 1] - first; }
  if (rows <= 0) return;
  const elem_t* w = pt.w + (is_b ? 0 : (int64_t)g * pt.n * pt.k);
  const int64_t x0 = is_b || perm ? 0 : g * pt.gx, y0 = is_b || perm ? 0 : g * pt.gy;
  const int steps = pt.k / KSTEP, s0 = steps * wave / KW, s1 = steps * (wave + 1) / KW;
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
      xp[m] = pt.x + (int64_t)(pair / div) * pt.ldx + x0 + FR * l4;
    }
    const int mb = min(MB, (rows - m0 + 15) >> 4);     // row blocks with work (uniform)
    f32x4 acc[NR][MB];
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int m = 0; m < MB; ++m) acc[r][m] = zero4();
    // two sets of U steps of weights in turn (HBM), two sets of two steps of x in turn (L1 / L2), each requested one set ahead
    frag_t wf[2][NR][U], xf[2][MB][2];
    auto request_w = [&](frag_t (&f)[NR][U], int s) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < NR; ++r) f[r][u] = __builtin_nontemporal_load((const frag_t*)(wp[r] + (int64_t)(s + u) * KSTEP));
    };
    auto request_x = [&](frag_t (&f)[MB][2], int s) {
#pragma unroll
      for (int m = 0; m < MB; ++m) {
        if (m < mb) {
          f[m][0] = *(const frag_t*)(xp[m] + (int64_t)s * KSTEP);
          f[m][1] = *(const frag_t*)(xp[m] + (int64_t)(s + 1) * KSTEP);
        }
      }
    };
    auto multiply = [&](frag_t (&f)[NR][U], int s) {
#pragma unroll
      for (int u = 0; u < U; u += 2) {
        if (s + u + 4 <= s1) request_x(xf[(u / 2 + 1) & 1], s + u + 2);
#pragma unroll
        for (int m = 0; m < MB; ++m) {
          if (m < mb) {
#pragma unroll
            for (int v = 0; v < 2; ++v)
#pragma unroll
              for (int r = 0; r < NR; ++r) acc[r][m] = mma(f[r][u + v], xf[(u / 2) & 1][m][v], acc[r][m]);
          }
        }
      }
    };
    int s = s0;
    if (s + U <= s1) {
      request_w(wf[0], s);
      request_x(xf[0], s);
      while (true) {
        if (s + 2 * U <= s1) request_w(wf[1], s + U);
        multiply(wf[0], s);
        s += U;
        if (s + U > s1) break;
        if (s + 2 * U <= s1) request_w(wf[0], s + U);
        multiply(wf[1], s);
        s += U;
        if (s + U > s1) break;
      }
    }
    for (; s < s1; ++s) {
      frag_t w1[NR];
#pragma unroll
      for (int r = 0; r < NR; ++r) w1[r] = *(const frag_t*)(wp[r] + (int64_t)s * KSTEP);
#pragma unroll
      for (int m = 0; m < MB; ++m) {
        if (m < mb) {
          const frag_t x1 = *(const frag_t*)(xp[m] + (int64_t)s * KSTEP);
#pragma unroll
          for (int r = 0; r < NR; ++r) acc[r][m] = mma(w1[r], x1, acc[r][m]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int m = 0; m < MB; ++m) *(f32x4*)&red[wave][16 * m + l15][16 * r + 4 * l4] = acc[r][m];
    __syncthreads();
    constexpr int OB = EPI == LM_EPI_GLU ? NR / 2 : NR;      // 16-channel blocks of the result
    for (int i = tid; i < 16 * MB * OB * 4; i += 64 * KW) {
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
      if (c < (EPI == LM_EPI_GLU ? pt.n / 2 : pt.n)) {
        if constexpr (EPI == LM_EPI_GLU) v = glu(pt, p.act, n0 + 16 * sb + c4, v, up);
        store4<EPI>(pt, pair, c, y0, v, p.scale);
      }
    }
    __syncthreads();
  }
}

constexpr int TM = LM_TILE_ROWS, TN = 128;                  // rows, channels of a tile
constexpr int SROWB = 64, SK = SROWB / (int)sizeof(elem_t);  // a stage: 64 bytes of k of every row
constexpr int STAGE = (TM + TN) * SROWB, STAGES = 3;
static_assert(TM == 256, "the wave layout");

// LDS rows of 64 bytes, four 16-byte slots and four rows to a 256-byte line: slot s of row r at s ^ (0, 2, 3, 1)[r / 4 % 4], with
// the property Tile::swizzle has for fragment reads
__device__ __forceinline__ int stage_swizzle(int row) {
  const int q = (row >> 2) & 3;
  return (((q ^ (q >> 1)) & 1) << 1) | (q >> 1);
}

// 4 waves, 128 rows x 64 channels each; three stages: while one multiplies, two are on their way
template <int EPI>
__global__ __launch_bounds__(256, 2) void gemm_tiles_kernel(GemmArgs p, int mt_a, int mt_b) {
  __shared__ __attribute__((aligned(16))) uint8_t lds[STAGES * STAGE];
  __shared__ int y_row[TM];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  // linear order: bands of row tiles, all channel tiles of a band before the next one; of both parts a contiguous range per XCD
  const int nt_a = (p.a.n + TN - 1) / TN, nt_b = mt_b ? (p.b.n + TN - 1) / TN : 0;
  const int wgs_b = 8 * ((mt_b * nt_b + 7) >> 3);
  const bool is_b = (int)blockIdx.x < wgs_b;
  const Part& pt = is_b ? p.b : p.a;
  const int nt = is_b ? nt_b : nt_a, mts = is_b ? mt_b : mt_a;
  const int id = xcd_contiguous(is_b ? blockIdx.x : blockIdx.x - wgs_b, mts * nt);
  if (id < 0) return;
  constexpr int GM = 4;
  const int band = id / (GM * nt), in = id - band * GM * nt, bm = min(GM, mts - band * GM);
  const int mi = band * GM + in % bm, ni = in / bm;
  const int* perm = is_b ? nullptr : p.perm;
  int first = mi * TM, rows, g = 0;
  if (perm) {
    const i32x4 t = *(const i32x4*)(p.tiles + 4 * mi);       // group, first place, rows
    if (t[2] <= 0) return;
    g = t[0];
    first = t[1];
    rows = t[2];
  } else {
    rows = min(TM, (is_b ? p.rows_b : p.rows_a) - first);
  }
  const int n0 = ni * TN;
  const elem_t* w = pt.w + (int64_t)g * pt.n * pt.k;
  // pieces of 16 rows: lane -> (row lane / 4, physical slot lane % 4); a wave carries 2 of the weights' and 4 of x's
  const elem_t *wsrc[2], *xsrc[4];
  const int pr = lane >> 2, ps = (lane & 3) ^ stage_swizzle(pr);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = min(16 * (4 * wave + i) + pr, rows - 1);
    const int xr = perm ? perm[first + r] / p.x_div : first + r;
    xsrc[i] = pt.x + (int64_t)xr * pt.ldx + ps * FR;
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) wsrc[i] = w + (int64_t)min(n0 + 16 * (2 * wave + i) + pr, pt.n - 1) * pt.k + ps * FR;
  y_row[tid] = tid < rows ? (perm ? perm[first + tid] : first + tid) : -1;
  const uint32_t lds0 = (uint32_t)(size_t)(__attribute__((address_space(3))) uint8_t*)lds;
  const int uw = __builtin_amdgcn_readfirstlane(wave);
  auto stage = [&](int st, int k0) {
    const uint32_t dst = lds0 + st * STAGE;
#pragma unroll
    for (int i = 0; i < 2; ++i) dma16_uncounted(wsrc[i] + k0, dst + 1024 * (2 * uw + i));
#pragma unroll
    for (int i = 0; i < 4; ++i) dma16_uncounted(xsrc[i] + k0, dst + TN * SROWB + 1024 * (4 * uw + i));
  };
  const int wn = 64 * (wave & 1), wm = 128 * (wave >> 1);
  f32x4 acc[4][8];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[i][j] = zero4();
  const int nk = pt.k / SK;                                 // (>= 2: k is a multiple of 64)
  const int lane_off = l15 * SROWB + ((l4 ^ stage_swizzle(l15)) << 4);
  wait_pieces<0>();                                         // the compiler's own loads
  stage(0, 0);
  stage(1, SK);
  int st = 0;
  for (int t = 0; t < nk; ++t) {
    if (t + 1 < nk) wait_pieces<6>();                       // stage t is there, the 6 pieces of t + 1 may still fly
    else wait_pieces<0>();
    __builtin_amdgcn_s_barrier();                           // ... for every wave, and everyone has left stage t - 1
    asm volatile("" ::: "memory");
    if (t + 2 < nk) stage(st == 0 ? 2 : st - 1, (t + 2) * SK);
    const uint8_t* wt = lds + st * STAGE + wn * SROWB + lane_off;
    const uint8_t* xt = lds + st * STAGE + (TN + wm) * SROWB + lane_off;
    frag_t a[4], b[8];
#pragma unroll
    for (int i = 0; i < 4; ++i) a[i] = *(const frag_t*)(wt + 16 * SROWB * i);
#pragma unroll
    for (int j = 0; j < 8; ++j) b[j] = *(const frag_t*)(xt + 16 * SROWB * j);
    __builtin_amdgcn_s_setprio(1);
#pragma unroll
    for (int j = 0; j < 8; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i][j] = mma(a[i], b[j], acc[i][j]);
    __builtin_amdgcn_s_setprio(0);
    st = st == 2 ? 0 : st + 1;
  }
  __syncthreads();                                          // the stages are free
  if constexpr (EPI == LM_EPI_F32) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int row = y_row[wm + 16 * j + l15];
      if (row < 0) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = n0 + wn + 16 * i + 4 * l4;
        if (c < pt.n) store4<EPI>(pt, row, c, 0, acc[i][j], p.scale);
      }
    }
  } else {
    // through LDS, so that a row leaves in whole 16-byte pieces of neighbouring lanes: 32 rows of the wave's at a time
    constexpr int OC = EPI == LM_EPI_GLU ? 32 : 64, PITCH = OC * (int)sizeof(elem_t) + 16, PPR = OC / FR;
    static_assert(4 * 32 * PITCH <= STAGES * STAGE, "the waves' buffers");
    uint8_t* buf = lds + wave * 32 * PITCH;
#pragma unroll
    for (int part = 0; part < 4; ++part) {
#pragma unroll
      for (int jj = 0; jj < 2; ++jj) {
        const int j = 2 * part + jj;
#pragma unroll
        for (int i = 0; i < 4; i += EPI == LM_EPI_GLU ? 2 : 1) {
          f32x4 v = acc[i][j];
          int c = 16 * i;
          if constexpr (EPI == LM_EPI_GLU) {
            c = 8 * i;
            if (n0 + wn + 16 * i < pt.n) v = glu(pt, p.act, n0 + wn + 16 * i + 4 * l4, v, acc[i + 1][j]);
          }
          *(quad_t*)(buf + (16 * jj + l15) * PITCH + (c + 4 * l4) * (int)sizeof(elem_t)) = to_quad(v);
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int i = 0; i < 32 * PPR / 64; ++i) {
        const int pc = 64 * i + lane, r = pc / PPR, q = pc % PPR;
        const int row = y_row[wm + 32 * part + r], c = (EPI == LM_EPI_GLU ? (n0 + wn) / 2 : n0 + wn) + q * FR;
        if (row >= 0 && c < (EPI == LM_EPI_GLU ? pt.n / 2 : pt.n))
          *(frag_t*)((elem_t*)pt.y + (int64_t)row * pt.ldy + c) = *(const frag_t*)(buf + r * PITCH + q * 16);
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
    }
  }
}

static int check_part(const Part& p, int epi, int act) {
  if (!p.w || !p.x || !p.y || p.n <= 0 || p.k <= 0 || p.k % 64 || p.n % 16 || p.ldx < p.k || p.ldx % FR || p.ldy % FR) return LM_EINVAL;
  if (epi == LM_EPI_GLU && (p.n % 32 || (act != LM_ACT_SILU && act != LM_ACT_GELU_TANH))) return LM_EINVAL;
  if (epi == LM_EPI_GATE && (!p.gate || p.ldg % 4)) return LM_EINVAL;
  if (p.gx % FR || p.gy % 4) return LM_EINVAL;
  return LM_OK;
}

static int fill(GemmArgs& a, const LmGemmPart* pa, const LmGemmPart* pb, int groups, const int* perm, const int* off, int rows_a,
                int rows_b, int x_div, float scale, int epi, int act) {
  auto conv = [](const LmGemmPart* s) {
    return Part{(const elem_t*)s->w, (const elem_t*)s->x, s->ldx, s->y, s->ldy, s->n, s->k, s->gx, s->gy, s->bias,
                (const elem_t*)s->gate, s->ldg};
  };
  if (!pa || groups <= 0 || x_div <= 0 || (perm && !off) || epi < 0 || epi > LM_EPI_GATE) return LM_EINVAL;
  a.a = conv(pa);
  a.b = pb ? conv(pb) : Part{};
  if (check_part(a.a, epi, act) || (pb && check_part(a.b, epi, act))) return LM_EINVAL;
  a.groups = groups; a.perm = perm; a.off = off; a.rows_a = rows_a; a.rows_b = pb ? rows_b : 0; a.x_div = perm ? x_div : 1;
  a.tiles = nullptr; a.scale = scale; a.act = act;
  return LM_OK;
}

template <int NR, int KW, int EPI>
static int launch_rows(const GemmArgs& a, int max_rows, int has_b, hipStream_t s) {
  const int n = has_b && a.b.n > a.a.n ? a.b.n : a.a.n;
  const int mb = max_rows <= 16 || (n <= 256 && !a.perm && max_rows <= 64) ? 1 : max_rows <= 32 ? 2 : 4;
  const dim3 grid((n + 16 * NR - 1) / (16 * NR), a.groups + has_b, a.perm ? 1 : (max_rows + 16 * mb - 1) / (16 * mb));
  const dim3 block(64 * KW);
  if (mb == 1) hipLaunchKernelGGL((gemm_rows_kernel<NR, 1, KW, EPI>), grid, block, 0, s, a);
  else if (mb == 2) hipLaunchKernelGGL((gemm_rows_kernel<NR, 2, KW, EPI>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((gemm_rows_kernel<NR, 4, KW, EPI>), grid, block, 0, s, a);
  return launch_status();
}

// Channels per workgroup: the more the fewer reads of x, as long as every CU has work.  A product of few channels over many rows
// (the router of a prompt) has its workgroups along the rows instead.
template <int EPI>
static int plan_rows(const GemmArgs& a, int max_rows, int has_b, hipStream_t s) {
  const int64_t n = (int64_t)a.groups * a.a.n;
  if constexpr (EPI == LM_EPI_GLU) {
    return n >= 64 * 256 ? launch_rows<4, 4, EPI>(a, max_rows, has_b, s) : launch_rows<2, 8, EPI>(a, max_rows, has_b, s);
  } else {
    if (max_rows > 64) return launch_rows<2, 8, EPI>(a, max_rows, has_b, s);
    if (n >= 64 * 512 || (n >= 64 * 150 && max_rows > 16)) return launch_rows<4, 4, EPI>(a, max_rows, has_b, s);
    if (n >= 64 * 150) return launch_rows<2, 4, EPI>(a, max_rows, has_b, s);
    return launch_rows<1, 8, EPI>(a, max_rows, has_b, s);
  }
}

}  // namespace lm

using namespace lm;

extern "C" int lm_gemm_rows(const LmGemmPart* pa, const LmGemmPart* pb, int groups, const int* perm, const int* off, int rows_a,
                            int rows_b, int x_div, int max_rows, float scale, int epi, int act, void* stream) {
  GemmArgs a;
  if (fill(a, pa, pb, groups, perm, off, rows_a, rows_b, x_div, scale, epi, act) || max_rows <= 0) return LM_EINVAL;
  hipStream_t s = (hipStream_t)stream;
  const int has_b = pb && rows_b > 0;
  if (epi == LM_EPI_GLU) return plan_rows<LM_EPI_GLU>(a, max_rows, has_b, s);
  if (epi == LM_EPI_GATE) return plan_rows<LM_EPI_GATE>(a, max_rows, has_b, s);
  return epi == LM_EPI_F32 ? plan_rows<LM_EPI_F32>(a, max_rows, has_b, s) : plan_rows<LM_EPI_ELEM>(a, max_rows, has_b, s);
}

extern "C" int lm_gemm_tiles(const LmGemmPart* pa, const LmGemmPart* pb, int groups, const int* perm, const int* off,
                             const int* tiles, int max_tiles, int rows_a, int rows_b, int x_div,
                             float scale, int epi, int act, void* stream) {
  GemmArgs a;
  if (fill(a, pa, pb, groups, perm, off, rows_a, rows_b, x_div, scale, epi, act)) return LM_EINVAL;
  if (epi == LM_EPI_GATE || (groups > 1 && !perm)) return LM_EINVAL;      // few rows only
  if (perm && (!tiles || max_tiles <= 0)) return LM_EINVAL;
  a.tiles = perm ? tiles : nullptr;
  const int mt_a = perm ? max_tiles : (rows_a + TM - 1) / TM, mt_b = pb && rows_b > 0 ? (rows_b + TM - 1) / TM : 0;
  const int64_t tiles_a = (int64_t)mt_a * ((a.a.n + TN - 1) / TN), tiles_b = mt_b ? (int64_t)mt_b * ((a.b.n + TN - 1) / TN) : 0;
  if (tiles_a <= 0 || tiles_a + tiles_b > (1 << 30)) return LM_EINVAL;
  const dim3 grid((unsigned)(8 * ((tiles_a + 7) / 8) + 8 * ((tiles_b + 7) / 8)));
  hipStream_t s = (hipStream_t)stream;
  if (epi == LM_EPI_ELEM) hipLaunchKernelGGL((gemm_tiles_kernel<LM_EPI_ELEM>), grid, dim3(256), 0, s, a, mt_a, mt_b);
  else if (epi == LM_EPI_F32) hipLaunchKernelGGL((gemm_tiles_kernel<LM_EPI_F32>), grid, dim3(256), 0, s, a, mt_a, mt_b);
  else hipLaunchKernelGGL((gemm_tiles_kernel<LM_EPI_GLU>), grid, dim3(256), 0, s, a, mt_a, mt_b);
  return launch_status();
}
