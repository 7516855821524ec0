// Latent attention: the cache holds one row per token, [normed latent c | turned key part], that all heads share.
//
//   lm_latent_append  prompt portions: norm + rotation of the row, stored in its page; the queries' turned parts in place.  (The
//                     portions' attention runs on keys and values expanded from the rows by a product: lm_attn_prefill.)
//   lm_latent_decode  one token per sequence: the queries' unturned parts have been taken into the latent space (W_uk^T q), so a
//                     cache row is key (all of it) and value (its latent) of every head.  A workgroup serves 16 or 32 heads, the
//                     columns of the MFMA tiles, and one part of the keys; its waves share the rows in LDS, divide the scores among
//                     themselves and own a quarter of the latent's columns each.
//   lm_gather_pages   the pages of the portions' contexts, one behind the other
#include "lm_attn.h"
#include "omniserve_lm.h"

namespace lm {

// The cache row of one token from its projection; the whole workgroup (256 threads or more), Rp <= 1024.
__device__ __forceinline__ void latent_row(const elem_t* src, const float* w, float eps, const float* freq, int half, int pos,
                                           elem_t* dst, int R, int Rp, int Tp, float* red) {
  const int tid = threadIdx.x, c = 4 * tid;
  const f32x4 v = c < Rp ? from_quad(*(const quad_t*)(src + c)) : zero4();      // (columns from R on are zero)
  const float ss = wave_sum((v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]));
  if ((tid & 63) == 0 && tid < 256) red[tid >> 6] = ss;
  __syncthreads();
  const float r = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)R + eps);
  if (c < Rp) *(quad_t*)(dst + c) = to_quad(v * r * *(const f32x4*)(w + c));
  if (tid < half) {
    float s, co;
    sincosf((float)pos * freq[tid], &s, &co);
    const float a = (float)src[Rp + tid], b = (float)src[Rp + half + tid];
    dst[Rp + tid] = (elem_t)(a * co - b * s);
    dst[Rp + half + tid] = (elem_t)(b * co + a * s);
  } else if (tid + half < Tp) {
    dst[Rp + half + tid] = (elem_t)0.f;
  }
}

struct LatentAppendArgs {
  elem_t* x; int64_t ld, src_col;       // row: q [H][dk], ..., from src_col on the projected cache row; src_col < 0: none
  const float* w; float eps;
  const float* freq; int half;
  const int *pos, *slot;
  elem_t* cache;                        // [pages][64][Rp + Tp]
  int H, dk, q_rot, R, Rp, Tp;
};

__global__ __launch_bounds__(256) void latent_append_kernel(LatentAppendArgs p) {
  __shared__ f32x2 cs[128];
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x, pos = p.pos[t], slot = p.slot[t];
  if (tid < p.half) {
    float s, c;
    sincosf((float)pos * p.freq[tid], &s, &c);
    cs[tid] = (f32x2){c, s};
  }
  __syncthreads();
  elem_t* row = p.x + (int64_t)t * p.ld;
  if (p.half % 4 == 0 && p.q_rot % 4 == 0) {
    const int nq = p.half / 4;
    for (int i = tid; i < p.H * nq; i += 256) {
      const int h = i / nq, d = 4 * (i - h * nq);
      quad_t* q = (quad_t*)(row + (int64_t)h * p.dk + p.q_rot + d);
      const f32x4 a = from_quad(q[0]), b = from_quad(q[nq]);
      f32x4 u, v;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        u[e] = a[e] * cs[d + e][0] - b[e] * cs[d + e][1];
        v[e] = b[e] * cs[d + e][0] + a[e] * cs[d + e][1];
      }
      q[0] = to_quad(u);
      q[nq] = to_quad(v);
    }
  } else for (int i = tid; i < p.H * p.half; i += 256) {
    const int h = i / p.half, d = i - h * p.half;
    elem_t* q = row + (int64_t)h * p.dk + p.q_rot + d;
    const float a = (float)q[0], b = (float)q[p.half];
    q[0] = (elem_t)(a * cs[d][0] - b * cs[d][1]);
    q[p.half] = (elem_t)(b * cs[d][0] + a * cs[d][1]);
  }
  if (p.src_col >= 0 && slot >= 0)
    latent_row(row + p.src_col, p.w, p.eps, p.freq, p.half, pos, p.cache + (int64_t)slot * (p.Rp + p.Tp), p.R, p.Rp, p.Tp, red);
}

__global__ __launch_bounds__(256) void gather_pages_kernel(frag_t* dst, const frag_t* src, const int* pages, int row_frags) {
  const int n = PAGE * row_frags;
  const frag_t* s = src + (int64_t)pages[blockIdx.x] * n;
  frag_t* d = dst + (int64_t)blockIdx.x * n;
  for (int i = threadIdx.x + 256 * blockIdx.y; i < n; i += 256 * gridDim.y) d[i] = s[i];
}

struct LatentDecodeArgs {
  const elem_t* x; int64_t ld, src_col;        // as above; the queries' turned parts are read as projected
  const float* w; float eps;
  const float* freq; int half;
  const int *pos, *slot;                       // pos < 0: an empty place of the batch
  elem_t* cache;
  const int* bt; int bt_stride;
  const elem_t* qa;                            // [B][H][RP]
  elem_t* o;                                   // [B][H][RP]
  float* part;                                 // nsplit > 1: [B][H][nsplit][RP + 2]
  float scale;                                 // includes log2(e)
  int nsplit, H, dk, q_rot, R;
};

// HB blocks of 16 heads share the tiles.  Of the scores of a tile (32 keys) each wave forms 16 keys x 16 heads; they meet in LDS.
// Of the values each wave owns a quarter of the columns, for all heads.
template <int RP, int TP, int HB>
struct LatentGeom {
  static constexpr int KT = 32, ROW = RP + TP, ES = (int)sizeof(elem_t);
  static constexpr int CB = KT * RP * ES, TB = KT * TP * ES, BUF = CB + TB;
  static constexpr int NP = BUF / 1024, P = (NP + 3) / 4;      // 1-KiB pieces of a tile, pieces per wave
  static constexpr int SP = KT * 4 + 16, QP = TP * ES;          // rows of the scores, of the turned queries (the same place)
  static constexpr int AUX = 16 * HB * (SP > QP ? SP : QP);
  static constexpr size_t LDS = 2 * BUF + AUX;
};

template <int RP, int TP, int HB>
__global__ __launch_bounds__(256, SPLIT ? 2 : 1) void latent_decode_kernel(LatentDecodeArgs p) {
  typedef LatentGeom<RP, TP, HB> Gm;
  typedef Tile<RP * (int)sizeof(elem_t)> CT;
  typedef Tile<TP * (int)sizeof(elem_t)> TT;
  constexpr int ROW = Gm::ROW, NCF = RP / KSTEP, NTF = TP / KSTEP, NVB = RP / 64;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];      // two key tiles, scores
  uint8_t* aux = lds + 2 * Gm::BUF;
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int b = blockIdx.x, h0 = 16 * HB * blockIdx.y, split = blockIdx.z;
  const int ub = wave & 1, hb = HB == 2 ? wave >> 1 : 0;            // scores: key block, head block
  const int pos = __builtin_amdgcn_readfirstlane(p.pos[b]);
  if (pos < 0) return;
  const int nt = pos / Gm::KT + 1, per = (nt + p.nsplit - 1) / p.nsplit, ta = split * per, tb = min(nt, ta + per);
  const int* bt = p.bt + (int64_t)b * p.bt_stride;
  const elem_t* row = p.x + (int64_t)b * p.ld;

  const uint32_t lds0 = (uint32_t)(size_t)(__attribute__((address_space(3))) uint8_t*)lds;
  const int uw = __builtin_amdgcn_readfirstlane(wave);
  // page numbers, 64 at a time, one per lane: the loop is to have no loads of its own
  const int last_page = pos / PAGE;
  int page0 = ta * Gm::KT / PAGE, pages = bt[min(page0 + lane, last_page)];
  auto stage = [&](int t) {      // every wave P pieces, the last one twice where they do not divide (equal bytes)
    const int kb = Gm::KT * t;
    if (kb / PAGE >= page0 + 64) {
      page0 += 64;
      pages = bt[min(page0 + lane, last_page)];
    }
    const elem_t* src = p.cache + ((int64_t)__builtin_amdgcn_readlane(pages, kb / PAGE - page0) * PAGE + kb % PAGE) * ROW;
    const uint32_t dst = lds0 + (uint32_t)((t - ta) & 1) * Gm::BUF;
#pragma unroll
    for (int i = 0; i < Gm::P; ++i) {
      const int pc = min(uw + 4 * i, Gm::NP - 1);
      const bool turned = pc >= Gm::CB / 1024;
      const int sc = pc * 64 + lane, st = sc - Gm::CB / 16;
      const uint32_t oc = (sc / CT::NS) * ROW + ((sc % CT::NS) ^ CT::swizzle(sc / CT::NS)) * FR;
      const uint32_t ot = (st / TT::NS) * ROW + RP + ((st % TT::NS) ^ TT::swizzle(st / TT::NS)) * FR;
      dma16_uncounted(src + (turned ? ot : oc), dst + 1024 * pc);
    }
  };
  static_assert(Gm::CB % 1024 == 0 && Gm::TB % 1024 == 0, "whole pieces");
  // queries: the latent part as it is, the turned part through LDS
  frag_t qf[NCF + NTF];
  const elem_t* qp = p.qa + ((int64_t)b * p.H + min(h0 + 16 * hb + l15, p.H - 1)) * RP + FR * l4;
#pragma unroll
  for (int s = 0; s < NCF; ++s) qf[s] = *(const frag_t*)(qp + s * KSTEP);
  constexpr int NQ = 16 * HB * (TP / 2) / 256;
  float qu[NQ], qv[NQ], qa[NQ];                        // pairs; those past `half` are padding
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    const int hh = (256 * i + tid) / (TP / 2), d = min((256 * i + tid) % (TP / 2), p.half - 1);
    const elem_t* q = row + (int64_t)min(h0 + hh, p.H - 1) * p.dk + p.q_rot + d;
    qu[i] = (float)q[0];
    qv[i] = (float)q[p.half];
    qa[i] = (float)pos * p.freq[d];
  }
  // The first tile is on its way while the rest is prepared (what the compiler loads behind it only makes the loop's first wait
  // stricter) -- but behind the new row where this workgroup brings it: every one whose part holds the newest tile writes the row
  // (equal bytes).
  const int slot = p.slot[b];
  const bool append = tb == nt && ta < tb && slot >= 0 && p.src_col >= 0;
  if (append) {
    latent_row(row + p.src_col, p.w, p.eps, p.freq, p.half, pos, p.cache + (int64_t)slot * ROW, p.R, RP, TP, red);
    __syncthreads();    // (makes it visible to the other waves of this workgroup)
  }
  if (ta < tb) stage(ta);
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    const int hh = (256 * i + tid) / (TP / 2), d = (256 * i + tid) % (TP / 2);
    const bool in = d < p.half && h0 + hh < p.H;
    float s, c;
    sincosf(qa[i], &s, &c);
    elem_t* q = (elem_t*)(aux + hh * Gm::QP);
    const int at = d < p.half ? d : 2 * p.half + 2 * (d - p.half);
    q[at] = in ? (elem_t)(qu[i] * c - qv[i] * s) : (elem_t)0.f;
    q[d < p.half ? d + p.half : at + 1] = in ? (elem_t)(qv[i] * c + qu[i] * s) : (elem_t)0.f;
  }
  f32x4 acc[HB][NVB];
  float m_run[HB], l_run[HB];
#pragma unroll
  for (int g = 0; g < HB; ++g) {
#pragma unroll
    for (int c = 0; c < NVB; ++c) acc[g][c] = zero4();
    m_run[g] = NEG;
    l_run[g] = 0.f;
  }
  __syncthreads();
#pragma unroll
  for (int s = 0; s < NTF; ++s) qf[NCF + s] = *(const frag_t*)(aux + (16 * hb + l15) * Gm::QP + (s * KSTEP + FR * l4) * Gm::ES);
  for (int t = ta; t < tb; ++t) {
    wait_pieces<0>();
    __syncthreads();                                   // tile t is there for every wave, and everyone has left tile t - 1
    if (t + 1 < tb) stage(t + 1);
    const uint8_t *ct = lds + ((t - ta) & 1) * Gm::BUF, *tt = ct + Gm::CB;
    const int kb = Gm::KT * t;
    if (HB == 2 || wave < 2) {
      f32x4 x = zero4(), y = zero4();                  // two chains of products
#pragma unroll
      for (int s = 0; s < NCF; s += 2) {
        x = mma(CT::frag(ct, 16 * ub + l15, 4 * s + l4), qf[s], x);
        y = mma(CT::frag(ct, 16 * ub + l15, 4 * s + 4 + l4), qf[s + 1], y);
      }
#pragma unroll
      for (int s = 0; s < NTF; s += 2) {
        x = mma(TT::frag(tt, 16 * ub + l15, 4 * s + l4), qf[NCF + s], x);
        y = mma(TT::frag(tt, 16 * ub + l15, 4 * s + 4 + l4), qf[NCF + s + 1], y);
      }
      x += y;
#pragma unroll
      for (int r = 0; r < 4; ++r) x[r] = kb + 16 * ub + 4 * l4 + r <= pos ? x[r] : NEG;
      *(f32x4*)(aux + (16 * hb + l15) * Gm::SP + (16 * ub + 4 * l4) * 4) = x;
    }
    __syncthreads();
    quad_t pq[HB][2][NOPND];
    float alpha[HB];
#pragma unroll
    for (int g = 0; g < HB; ++g) {
      f32x4 x[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) x[u] = *(const f32x4*)(aux + (16 * g + l15) * Gm::SP + (16 * u + 4 * l4) * 4);
      alpha[g] = softmax_step<2>(x, p.scale, m_run[g], l_run[g], pq[g]);
      if (__builtin_amdgcn_ballot_w64(alpha[g] != 1.0f) != 0) {
#pragma unroll
        for (int c = 0; c < NVB; ++c) acc[g][c] *= alpha[g];
      }
    }
#pragma unroll
    for (int c = 0; c < NVB; ++c) {
      const quad_t v0 = CT::column_quad(ct, 0, wave * NVB + c, l15, l4), v1 = CT::column_quad(ct, 16, wave * NVB + c, l15, l4);
#pragma unroll
      for (int g = 0; g < HB; ++g)
#pragma unroll
        for (int o = 0; o < NOPND; ++o) acc[g][c] = mma_quads(v0, v1, pq[g][0][o], pq[g][1][o], acc[g][c]);
    }
  }
#pragma unroll
  for (int g = 0; g < HB; ++g) {
    const float l = column_sum(l_run[g]);
    const int h = h0 + 16 * g + l15;
    if (h >= p.H) continue;
    const int64_t hrow = (int64_t)b * p.H + h;
    if (p.nsplit > 1) {
      float* q = p.part + (hrow * p.nsplit + split) * (RP + 2);
      if (wave == 0 && l4 == 0) { q[0] = m_run[g]; q[1] = l; }
#pragma unroll
      for (int c = 0; c < NVB; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) q[2 + 16 * (wave * NVB + c) + 4 * l4 + r] = acc[g][c][r];
    } else {
      const float inv = 1.0f / l;
#pragma unroll
      for (int c = 0; c < NVB; ++c) *(quad_t*)(p.o + hrow * RP + 16 * (wave * NVB + c) + 4 * l4) = to_quad(acc[g][c] * inv);
    }
  }
}

template <int RP, int TP, int HB>
static int launch_blocks(const LatentDecodeArgs& a, int B, hipStream_t s) {
  auto k = latent_decode_kernel<RP, TP, HB>;
  constexpr size_t lds = LatentGeom<RP, TP, HB>::LDS;
  if (allow_lds(k, lds)) return LM_EINVAL;
  hipLaunchKernelGGL(k, dim3(B, (a.H + 16 * HB - 1) / (16 * HB), a.nsplit), dim3(256), lds, s, a);
  if (a.nsplit > 1)
    hipLaunchKernelGGL(attn_merge_kernel, dim3(B, a.H), dim3(256), 0, s, a.part, a.nsplit, a.pos, (const elem_t*)nullptr, (int64_t)0, a.o,
                       (int64_t)a.H * RP, a.H, RP);
  return launch_status();
}

template <int RP, int TP>
static int launch(const LatentDecodeArgs& a, int B, hipStream_t s) {
  return a.H > 16 ? launch_blocks<RP, TP, 2>(a, B, s) : launch_blocks<RP, TP, 1>(a, B, s);
}

static int check(int64_t ld, int64_t src_col, const float* w, int half, int H, int dk, int q_rot, int R, int Rp, int Tp) {
  if (H <= 0 || half < 0 || 2 * half > Tp || Tp > 256 || q_rot < 0 || q_rot + 2 * half > dk || R <= 0 || R > Rp || Rp % 64 || Rp > 1024 ||
      Tp % 64 || ld % FR || (src_col >= 0 && (!w || src_col % FR)))
    return LM_EINVAL;
  return LM_OK;
}

}  // namespace lm

using namespace lm;

extern "C" int lm_latent_append(void* x, int64_t ld, int64_t src_col, const float* w, float eps, const float* freq, int half,
                                const int* pos, const int* slot, void* cache, int tokens, int H, int dk, int q_rot, int R, int Rp, int Tp,
                                void* stream) {
  if (tokens <= 0 || check(ld, src_col, w, half, H, dk, q_rot, R, Rp, Tp)) return LM_EINVAL;
  LatentAppendArgs a{(elem_t*)x, ld, src_col, w, eps, freq, half, pos, slot, (elem_t*)cache, H, dk, q_rot, R, Rp, Tp};
  hipLaunchKernelGGL(latent_append_kernel, dim3(tokens), dim3(256), 0, (hipStream_t)stream, a);
  return launch_status();
}

extern "C" int lm_gather_pages(void* dst, const void* src, const int* pages, int n_pages, int row, void* stream) {
  if (n_pages <= 0 || row <= 0 || row % FR) return LM_EINVAL;
  hipLaunchKernelGGL(gather_pages_kernel, dim3(n_pages, 4), dim3(256), 0, (hipStream_t)stream, (frag_t*)dst, (const frag_t*)src, pages,
                     row / FR);
  return launch_status();
}

extern "C" int lm_latent_decode(const void* x, int64_t ld, int64_t src_col, const float* w, float eps, const float* freq, int half,
                                const int* pos, const int* slot, void* cache, const int* bt, int bt_stride, const void* qa, void* o,
                                float* part, int nsplit, float scale, int B, int H, int dk, int q_rot, int R, int Rp, int Tp,
                                void* stream) {
  if (B <= 0 || nsplit <= 0 || nsplit > 64 || (nsplit > 1 && !part) || !(scale > 0.f) ||
      check(ld, src_col, w, half, H, dk, q_rot, R, Rp, Tp))
    return LM_EINVAL;
  LatentDecodeArgs a{(const elem_t*)x, ld, src_col, w, eps, freq, half, pos, slot, (elem_t*)cache, bt, bt_stride, (const elem_t*)qa,
                     (elem_t*)o, part, scale * LOG2E, nsplit, H, dk, q_rot, R};
  hipStream_t s = (hipStream_t)stream;
#define LM_CASE(K, V) if (Rp == K && Tp == V) return launch<K, V>(a, B, s);
  LM_CASE(64, 64) LM_CASE(128, 64) LM_CASE(256, 64) LM_CASE(512, 64) LM_CASE(64, 128) LM_CASE(128, 128) LM_CASE(256, 128)
  LM_CASE(512, 128)
#undef LM_CASE
  return LM_EINVAL;
}
