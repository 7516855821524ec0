// Causal attention of prompt portions over the paged cache, with a sliding window, any grouping of query heads and separate
// key / value sizes.  One workgroup per (64 or 128 query rows, head): its waves share the K and V tiles (64 keys = one cache
// page) in LDS, brought by LDS-DMA into two buffers; only pages that some row of the workgroup can see are touched.  The output
// is multiplied with sigmoid(gate) before it is stored.
#include "lm_attn.h"
#include "omniserve_lm.h"

namespace lm {

struct AttnArgs {
  const elem_t* q; int64_t ldq;                // [tokens][H][dk]
  const elem_t* kc; int64_t k_page; int k_head, k_row;      // key i of head g in page p: kc + p k_page + g k_head + i k_row
  const elem_t* vc; int64_t v_page; int v_head, v_row;
  const int* bt; int bt_stride;                // page numbers, one row per entry
  const int* entry;                            // [entries][4]: first token, tokens, position of the first token, block table row
  const int* tiles; int n_tiles;               // [n_tiles][2]: entry, first row within the entry
  const elem_t* gate; int64_t ldg;             // [tokens][H][dv] or null
  elem_t* o; int64_t ldo;
  float scale;                                 // includes log2(e)
  int window, H, G;
};

constexpr int attn_waves_per_simd(int dk, int dv) { return SPLIT && dk + dv <= 256 ? 4 : 2; }      // what the registers allow

template <int DK, int DV, int WAVES>
struct AttnGeom {
  static constexpr int KB = DK * (int)sizeof(elem_t), VB = DV * (int)sizeof(elem_t);
  static constexpr bool DB = 2 * PAGE * (KB + VB) <= 131072 && SPLIT;          // two buffers
};

template <int DK, int DV, int WAVES>
__global__ __launch_bounds__(64 * WAVES, attn_waves_per_simd(DK, DV)) void attn_prefill_kernel(AttnArgs p) {
  typedef AttnGeom<DK, DV, WAVES> Gm;
  typedef Tile<Gm::KB> KT;
  typedef Tile<Gm::VB> VT;
  constexpr int NKF = DK / KSTEP, NVB = DV / 16;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int gs = p.H / p.G;
  const int id = xcd_contiguous(blockIdx.x, p.n_tiles * p.H);
  if (id < 0) return;
  const int u_ = id % gs, tile = id / gs % p.n_tiles, g = id / (gs * p.n_tiles), h = g * gs + u_;     // a kv head's work stays together
  const int e = p.tiles[2 * tile], row0 = p.tiles[2 * tile + 1];
  const int start = p.entry[4 * e], count = p.entry[4 * e + 1], pos0 = p.entry[4 * e + 2];
  const int* bt = p.bt + (int64_t)p.entry[4 * e + 3] * p.bt_stride;
  const int r_w = row0 + 16 * wave;                      // the wave's first row
  const int row = r_w + l15, rowc = min(row, count - 1);
  const int qpos = pos0 + rowc;
  const int wg_last = pos0 + min(row0 + 16 * WAVES, count) - 1;
  const int w_first = pos0 + min(r_w, count - 1), w_last = pos0 + min(r_w + 15, count - 1);
  const bool idle = r_w >= count;

  frag_t qf[NKF];
  {
    const elem_t* qp = p.q + (int64_t)(start + rowc) * p.ldq + (int64_t)h * DK + FR * l4;
#pragma unroll
    for (int s = 0; s < NKF; ++s) qf[s] = *(const frag_t*)(qp + s * KSTEP);
  }
  f32x4 acc[NVB];
#pragma unroll
  for (int c = 0; c < NVB; ++c) acc[c] = zero4();
  float m_run = NEG, l_run = 0.f;

  const int lo = max(0, pos0 + row0 - p.window + 1);     // first key the workgroup needs
  const int kb0 = lo & ~(PAGE - 1);
  const int k_rowb = p.k_row * (int)sizeof(elem_t), v_rowb = p.v_row * (int)sizeof(elem_t);
  // 1-KiB pieces of a tile, one per wave and turn; physical slot s of row r holds logical slot s ^ swizzle(r)
  auto bring = [&](auto tile, const uint8_t* src, int rowb, uint8_t* dst) {
    typedef decltype(tile) T;
    constexpr int ROWB = T::NS * 16, N = PAGE * ROWB / 1024, STEP = 1024 * WAVES / ROWB;
    constexpr bool EVEN = 1024 * WAVES % ROWB == 0 && STEP % 16 == 0;      // every turn's rows have the first one's swizzles
#pragma unroll
    for (int i = 0; i < (N + WAVES - 1) / WAVES; ++i) {
      const int pc = wave + WAVES * i;
      if (N % WAVES != 0 && pc >= N) continue;
      const int sl = (EVEN ? wave : pc) * 64 + lane, r = sl / T::NS, s = sl % T::NS;
      const uint32_t off = r * rowb + ((s ^ T::swizzle(r)) << 4);
      dma16(src + (EVEN ? i * STEP * rowb : 0) + off, dst + 1024 * pc);
    }
  };
  auto stage = [&](int kb, uint8_t* kt, uint8_t* vt) {
    const int64_t page = bt[kb / PAGE];
    bring(KT{}, (const uint8_t*)(p.kc + page * p.k_page + g * p.k_head), k_rowb, kt);
    bring(VT{}, (const uint8_t*)(p.vc + page * p.v_page + g * p.v_head), v_rowb, vt);
  };
  auto compute = [&](int kb, const uint8_t* kt, const uint8_t* vt, auto prefetch) {
    const bool skip = idle || kb > w_last || kb + PAGE - 1 <= w_first - p.window;      // nothing visible for this wave
    f32x4 x[4];
    if (!skip) {
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        x[u] = zero4();
#pragma unroll
        for (int s = 0; s < NKF; ++s) x[u] = mma(KT::frag(kt, 16 * u + l15, 4 * s + l4), qf[s], x[u]);
      }
      __builtin_amdgcn_s_setprio(0);
    }
    prefetch();
    if (skip) return;
    if (!(kb + PAGE - 1 <= w_first && kb > w_last - p.window)) {
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = kb + 16 * u + 4 * l4 + r;
          const int ok = (int)(key <= qpos) & (int)(key > qpos - p.window);
          x[u][r] = ok ? x[u][r] : NEG;
        }
    }
    quad_t pq[4][NOPND];
    const float alpha = softmax_step<4>(x, p.scale, m_run, l_run, pq);
    if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
      for (int c = 0; c < NVB; ++c) acc[c] *= alpha;
    }
    __builtin_amdgcn_s_setprio(1);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int c = 0; c < NVB; ++c) {
        const quad_t v0 = VT::column_quad(vt, 32 * kk, c, l15, l4), v1 = VT::column_quad(vt, 32 * kk + 16, c, l15, l4);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) acc[c] = mma_quads(v0, v1, pq[2 * kk][o], pq[2 * kk + 1][o], acc[c]);
      }
    __builtin_amdgcn_s_setprio(0);
  };

  uint8_t *kt0 = lds, *vt0 = lds + PAGE * Gm::KB;
  if constexpr (Gm::DB) {
    uint8_t *kt1 = vt0 + PAGE * Gm::VB, *vt1 = kt1 + PAGE * Gm::KB;
    stage(kb0, kt0, vt0);
    __syncthreads();
    for (int kb = kb0; kb <= wg_last; kb += 2 * PAGE) {
      compute(kb, kt0, vt0, [&] { if (kb + PAGE <= wg_last) stage(kb + PAGE, kt1, vt1); });
      __syncthreads();
      if (kb + PAGE > wg_last) break;
      compute(kb + PAGE, kt1, vt1, [&] { if (kb + 2 * PAGE <= wg_last) stage(kb + 2 * PAGE, kt0, vt0); });
      __syncthreads();
    }
  } else {
    for (int kb = kb0; kb <= wg_last; kb += PAGE) {
      stage(kb, kt0, vt0);
      __syncthreads();
      compute(kb, kt0, vt0, [] {});
      __syncthreads();
    }
  }
  const float inv = 1.0f / column_sum(l_run);
  if (row >= count) return;
  elem_t* op = p.o + (int64_t)(start + row) * p.ldo + (int64_t)h * DV + 4 * l4;
  const elem_t* gp = p.gate ? p.gate + (int64_t)(start + row) * p.ldg + (int64_t)h * DV + 4 * l4 : nullptr;
#pragma unroll
  for (int c = 0; c < NVB; ++c) {
    f32x4 y = acc[c] * inv;
    if (gp) {
      const f32x4 z = from_quad(*(const quad_t*)(gp + 16 * c));
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] *= sigmoid(z[r]);
    }
    *(quad_t*)(op + 16 * c) = to_quad(y);
  }
}

template <int DK, int DV>
static int launch(const AttnArgs& a, hipStream_t s) {
  constexpr int WAVES = LM_ATTN_ROWS / 16;
  typedef AttnGeom<DK, DV, WAVES> Gm;
  constexpr size_t lds = (size_t)PAGE * (Gm::KB + Gm::VB) * (Gm::DB ? 2 : 1);
  auto k = attn_prefill_kernel<DK, DV, WAVES>;
  if (allow_lds(k, lds)) return LM_EINVAL;
  const int64_t total = (int64_t)a.n_tiles * a.H;
  hipLaunchKernelGGL(k, dim3((unsigned)(8 * ((total + 7) / 8))), dim3(64 * WAVES), lds, s, a);
  return launch_status();
}

}  // namespace lm

using namespace lm;

extern "C" int lm_attn_prefill(const void* q, int64_t ldq, const void* kc, int64_t k_page, int k_head, int k_row,
                               const void* vc, int64_t v_page, int v_head, int v_row, const int* bt, int bt_stride, const int* entry, const int* tiles, int n_tiles, const void* gate, int64_t ldg, void* o, int64_t ldo,
                               float scale, int window, int H, int G, int dk, int dv, void* stream) {
  if (n_tiles <= 0 || G <= 0 || H % G || !(scale > 0.f) || window <= 0 || ldq % FR || ldo % 4 || ldg % 4 ||
      k_page % FR || k_head % FR || k_row % FR || v_page % FR || v_head % FR || v_row % FR ||
      k_row <= 0 || v_row <= 0 || k_row > (1 << 22) || v_row > (1 << 22) ||
      (int64_t)n_tiles * H > (1 << 28))
    return LM_EINVAL;
  AttnArgs a{(const elem_t*)q, ldq, (const elem_t*)kc, k_page, k_head, k_row, (const elem_t*)vc, v_page, v_head, v_row, bt, bt_stride, entry, tiles, n_tiles, (const elem_t*)gate,
             ldg, (elem_t*)o, ldo, scale * 1.4426950408889634f, window, H, G};
  hipStream_t s = (hipStream_t)stream;
#define LM_CASE(K, V) if (dk == K && dv == V) return launch<K, V>(a, s);
  LM_CASE(64, 64) LM_CASE(64, 128) LM_CASE(64, 256) LM_CASE(128, 64) LM_CASE(128, 128) LM_CASE(128, 256)
  LM_CASE(192, 64) LM_CASE(192, 128) LM_CASE(192, 256) LM_CASE(256, 64) LM_CASE(256, 128) LM_CASE(256, 256)
#undef LM_CASE
  return LM_EINVAL;
}
