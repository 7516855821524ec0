// Gated linear attention  S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,  o_t = scale S_t^T q_t  (per head; S f32 [dk][dv], one slot per
// sequence; alpha_t = sigmoid(a2 low_t + bias)^(1 / tau), one decay per key channel).
//
// Prompt portions, chunks of at most C tokens: with B_i = sum of log alpha from the chunk's start up to and with token i,
//     q'_i = q_i e^(B_i),  k'_j = k_j e^(-B_j)          o_i = S^T q'_i + sum_{j <= i} (q'_i . k'_j) v_j
//     S'   = e^(B_n) (S + sum_j k'_j v_j^T)
// e^(-B) grows with strong decays, so a chunk ends in front of the first token that takes some channel's -B over LIMIT: everything
// stays within f32 whatever the decays are, and no term is lost (relative precision is that of f32).  A workgroup owns 64 or 128
// value columns of one head and walks the chunks of one segment; S stays in MFMA accumulators (16 columns per wave).  The decays'
// product a2 low is part of the chunk.  f32 factors (q', k', S, scores) enter the bf16 products as two bf16 operands each; of two
// such factors the product of the two low parts is dropped.
// Long portions are cut into segments that run in parallel: a first pass forms what each segment adds to the state and its total
// decay, the second starts every segment from the decayed sum of those before it.
#include "lm_state.h"
#include "omniserve_lm.h"

namespace lm {

constexpr float LIMIT = 40.0f;           // of -B, in powers of two

struct GlaArgs {
  const elem_t* x; int64_t ld;           // row: q [H][dk], k [H][dk], v [H][dv], ...; from low_col on the decays' low-rank input
  elem_t* o; int64_t ldo;                // [tokens][H][dv]
  float* state;                          // [slots][H][dk][dv]
  float* seg_state;                      // [segments][H][dk * dv]
  float* seg_decay;                      // [segments][H][dk], powers of two
  const int* seg;                        // [segments][8]: first token, tokens, slot, 1 = starts from zero, index in its entry,
                                         //                segments of the entry, 0, 0
  int64_t low_col;
  const elem_t* a2; const float* bias;   // [H * dk][rp], [H * dk]
  int rp;
  float inv_tau, scale;
  int H, dv;
};

// log2 of one token's decay
__device__ __forceinline__ float log_decay(float z, float inv_tau) { return fmaxf(-softplus(-z) * (inv_tau * LOG2E), -LIMIT); }

template <int DK, int NWV>
struct GlaGeom {
  static constexpr int TH = 64 * NWV, DVB = 16 * NWV;
  static constexpr int C = 32;                                         // tokens per chunk
  static constexpr int ES = (int)sizeof(elem_t), KB = DK * ES, VB = DVB * ES;
  static constexpr int PB = C * ES + 16, BB = DK * 4 + 16;             // rows of the score matrix and of B
  static constexpr int Q0 = 0, K0 = Q0 + NOPND * C * KB, V0 = K0 + NOPND * C * KB, P0 = V0 + C * VB, B0 = P0 + NOPND * C * PB,
                       T0 = B0 + C * BB, LDS = T0 + DK * 4;
  static constexpr int NQ = (C * KB / 16 + TH - 1) / TH, NV = C * VB / (16 * TH);      // 16-byte loads per thread
  static constexpr bool QWHOLE = C * KB / 16 % TH == 0;
  static_assert(NV >= 1 && C * VB % (16 * TH) == 0, "value tile");
};

constexpr int gla_waves_per_simd(int dk, int waves) { return !SPLIT ? 1 : dk <= 128 ? (waves == 8 ? 4 : 2) : 1; }      // what the registers allow

template <int DK, int NWV, bool OUTPUT>
__global__ __launch_bounds__(64 * NWV, gla_waves_per_simd(DK, NWV)) void gla_prefill_kernel(GlaArgs p) {
  typedef GlaGeom<DK, NWV> Gm;
  typedef Tile<Gm::KB> KT;
  typedef Tile<Gm::VB> VT;
  constexpr int C = Gm::C, NS = DK / 16, RT = C / 16;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  uint8_t *qt = lds + Gm::Q0, *kt = lds + Gm::K0, *vt = lds + Gm::V0, *pt = lds + Gm::P0, *bb = lds + Gm::B0;
  float* tot = (float*)(lds + Gm::T0);
  __shared__ int ends[NWV];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int sg = blockIdx.x, h = blockIdx.y, dv0 = Gm::DVB * blockIdx.z;
  const int* sp = p.seg + 8 * sg;
  const int row0 = sp[0], count = sp[1], slot = sp[2], fresh = sp[3], idx = sp[4], nseg = sp[5];
  if (!OUTPUT && idx == nseg - 1) return;             // nothing follows the last segment
  const int64_t st_stride = (int64_t)DK * p.dv;
  const uint32_t sbase = 4 * l4 * p.dv + dv0 + 16 * wave + l15;     // this lane's column, row 4 l4
  auto store_state = [&](float* s, const f32x4 (&S)[NS]) {
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) s[sbase + (uint32_t)((16 * t + r) * p.dv)] = S[t][r];
  };
  auto load_state = [&](const float* s, f32x4 (&S)[NS]) {
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t][r] = s[sbase + (uint32_t)((16 * t + r) * p.dv)];
  };
  f32x4 S[NS];
#pragma unroll
  for (int t = 0; t < NS; ++t) S[t] = zero4();
  float* own = p.state + ((int64_t)slot * p.H + h) * st_stride;
  // states between the passes lie as the accumulators hold them: [segment][head][16 columns][NS][lane][4]
  auto seg_at = [&](int i) {
    return (f32x4*)(p.seg_state + ((int64_t)(sg - idx + i) * p.H + h) * st_stride + (int64_t)(dv0 + 16 * wave) * DK) + lane;
  };
  auto keep = [&](int i) {
    f32x4* s = seg_at(i);
#pragma unroll
    for (int t = 0; t < NS; ++t) s[64 * t] = S[t];
  };
  auto recall = [&](int i) {
    const f32x4* s = seg_at(i);
#pragma unroll
    for (int t = 0; t < NS; ++t) S[t] = s[64 * t];
  };
  if (idx == 0) {
    if (OUTPUT && nseg > 1) recall(nseg - 1);         // kept by the first pass: the last segment replaces the slot's state
    else if (!fresh) load_state(own, S);
    if (!OUTPUT) keep(nseg - 1);
  } else if (OUTPUT) {
    // ((s_0 d_1 + s_1) d_2 + s_2) ..., d the segments' decays
    recall(0);
    for (int i = 1; i < idx; ++i) {
      const float* d = p.seg_decay + ((int64_t)(sg - idx + i) * p.H + h) * DK + 4 * l4;
      const f32x4* s = seg_at(i);
      constexpr int B = NS < 4 ? NS : 4;
#pragma unroll
      for (int t0 = 0; t0 < NS; t0 += B) {
        f32x4 f[B], a[B];
#pragma unroll
        for (int t = 0; t < B; ++t) {
          f[t] = *(const f32x4*)(d + 16 * (t0 + t));
          a[t] = s[64 * (t0 + t)];
        }
#pragma unroll
        for (int t = 0; t < B; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) S[t0 + t][r] = S[t0 + t][r] * __builtin_amdgcn_exp2f(f[t][r]) + a[t][r];
      }
    }
  }

  const elem_t* src = p.x + (int64_t)row0 * p.ld;
  const int64_t qo = (int64_t)h * DK, ko = (int64_t)(p.H + h) * DK, vo = (int64_t)2 * p.H * DK + (int64_t)h * p.dv + dv0;
  frag_t rq[OUTPUT ? Gm::NQ : 1], rk[Gm::NQ], rv[Gm::NV];
  const int ldx = (int)p.ld;
  auto fetch = [&](int c0) {                           // (rows past the end: the last one's values meet k' = q' = 0)
    const elem_t* base = src + (int64_t)c0 * p.ld;     // the same for all lanes; the lanes' offsets fit 32 bits
    const int last = count - 1 - c0;
#pragma unroll
    for (int i = 0; i < Gm::NQ; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / KT::NS, s = sl % KT::NS;
      const uint32_t off = min(r, last) * ldx + s * FR;
      if constexpr (OUTPUT) rq[i] = *(const frag_t*)(base + qo + off);
      rk[i] = *(const frag_t*)(base + ko + off);
    }
#pragma unroll
    for (int i = 0; i < Gm::NV; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / VT::NS, s = sl % VT::NS;
      rv[i] = *(const frag_t*)(base + vo + (uint32_t)(min(r, last) * ldx + s * FR));
    }
  };
  // the decays' input: its first 64 columns (all of them, as a rule) are requested one chunk ahead
  constexpr int NL = 64 / KSTEP;
  frag_t rl[RT][NL];
  auto fetch_low = [&](int c0) {
    const elem_t* base = src + (int64_t)c0 * p.ld + p.low_col;
    const int last = count - 1 - c0;
#pragma unroll
    for (int u = 0; u < RT; ++u)
#pragma unroll
      for (int s = 0; s < NL; ++s) rl[u][s] = *(const frag_t*)(base + (uint32_t)(min(16 * u + l15, last) * ldx + s * KSTEP + FR * l4));
  };
  float total = 0.f;                                  // !OUTPUT: of channel tid, the segment's decay so far
  fetch_low(0);
  fetch(0);
  typename KT::Offsets at(l15, l4);
  for (int c0 = 0, n; c0 < count; c0 += n) {
    at.forget();
    // ---- B: tokens are the rows, channels the columns of the product tiles ----
    int end = C;                                      // first place whose B is below the limit
#pragma unroll 1
    for (int cb = wave; cb < NS; cb += NWV) {
      uint32_t ch = 16 * cb + l15;
      asm volatile("" : "+v"(ch));                    // (no addresses kept from chunk to chunk)
      const elem_t* ap = p.a2 + (int64_t)h * DK * p.rp;
      const uint32_t ao = ch * p.rp + FR * l4;
      frag_t a[64 / KSTEP];
#pragma unroll
      for (int s = 0; s < 64 / KSTEP; ++s) a[s] = *(const frag_t*)(ap + (ao + s * KSTEP));
      const float bias = (p.bias + h * DK)[ch];
      float carry = 0.f;
#pragma unroll
      for (int u = 0; u < RT; ++u) {
        f32x4 z = zero4();
#pragma unroll
        for (int s = 0; s < 64 / KSTEP; ++s) z = mma(rl[u][s], a[s], z);
        for (int s = 64; s < p.rp; s += KSTEP)
          z = mma(*(const frag_t*)(src + (int64_t)c0 * p.ld + p.low_col + (uint32_t)(min(16 * u + l15, count - 1 - c0) * ldx + s + FR * l4)),
                  *(const frag_t*)(ap + (ao + s)), z);
        float sum = 0.f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sum += log_decay(z[r] + bias, p.inv_tau);   // (places past the end follow all others and are not used)
          z[r] = sum;                                 // running sum within the lane
        }
        float before = 0.f, all = 0.f;                // of the lanes in front, of the block
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const float v = __shfl(sum, 16 * g + l15, 64);
          before += g < l4 ? v : 0.f;
          all += v;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * u + 4 * l4 + r;
          *(float*)(bb + i * Gm::BB + (16 * cb + l15) * 4) = z[r] + (before + carry);
        }
        carry += all;
      }
      if (__builtin_amdgcn_ballot_w64(carry < -LIMIT) != 0) {      // some channel's B passes the limit (B only falls)
#pragma unroll 1
        for (int i = C - 1; i >= 0; --i)
          if (__builtin_amdgcn_ballot_w64(*(const float*)(bb + i * Gm::BB + (16 * cb + l15) * 4) < -LIMIT) != 0) end = min(end, i);
      }
    }
    if (lane == 0) ends[wave] = end;
    __syncthreads();
    n = min(C, count - c0);
#pragma unroll
    for (int w = 0; w < NWV; ++w) n = min(n, ends[w]);
    n = max(n, 1);                                    // (a single token stays within the limit)

    // ---- q', k', v ----
#pragma unroll
    for (int i = 0; i < Gm::NQ; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / KT::NS, s = sl % KT::NS;
      if (!Gm::QWHOLE && r >= C) break;
      const float* B = (const float*)(bb + r * Gm::BB) + s * FR;
      const bool in = r < n;
      frag_t q[NOPND], k[NOPND];
#pragma unroll
      for (int e = 0; e < FR; ++e) {
        const float b = in ? B[e] : 0.f;
        const float kk = in ? (float)rk[i][e] * __builtin_amdgcn_exp2f(-b) : 0.f;
        k[0][e] = (elem_t)kk;
        if constexpr (SPLIT) k[NOPND - 1][e] = (elem_t)(kk - (float)k[0][e]);
        if constexpr (OUTPUT) {
          const float qq = in ? (float)rq[i][e] * p.scale * __builtin_amdgcn_exp2f(b) : 0.f;
          q[0][e] = (elem_t)qq;
          if constexpr (SPLIT) q[NOPND - 1][e] = (elem_t)(qq - (float)q[0][e]);
        }
      }
      const int off = KT::slot(r, s);
#pragma unroll
      for (int o = 0; o < NOPND; ++o) {
        *(frag_t*)(kt + o * C * Gm::KB + off) = k[o];
        if constexpr (OUTPUT) *(frag_t*)(qt + o * C * Gm::KB + off) = q[o];
      }
    }
#pragma unroll
    for (int i = 0; i < Gm::NV; ++i) {
      const int sl = Gm::TH * i + tid;
      *(frag_t*)(vt + VT::slot(sl / VT::NS, sl % VT::NS)) = rv[i];
    }
    if (tid < DK) {
      const float b = *(const float*)(bb + (n - 1) * Gm::BB + tid * 4);
      tot[tid] = __builtin_amdgcn_exp2f(b);
      total += b;
    }
    __syncthreads();

    quad_t vq[RT];                                     // V, column l15 of this wave, all tokens of the chunk
#pragma unroll
    for (int u = 0; u < RT; ++u) vq[u] = VT::column_quad(vt, 16 * u, wave, l15, l4);
    if constexpr (OUTPUT) {
      // scores (transposed product: column = row i of the score matrix), blocks (row it, key u) go round the waves
#pragma unroll
      for (int bi = 0; bi < (RT * RT + NWV - 1) / NWV; ++bi) {
        const int blk = bi * NWV + wave, it = blk % RT, u = blk / RT;
        if (u >= RT) continue;
        const int i = 16 * it + l15;
        f32x4 s = zero4();
        if (u <= it) {
#pragma unroll
          for (int k = 0; k < DK / KSTEP; ++k) {
            const frag_t k0 = KT::frag(kt, at, 16 * u, k), q0 = KT::frag(qt, at, 16 * it, k);
            s = mma(k0, q0, s);
            if constexpr (SPLIT) {
              s = mma(k0, KT::frag(qt + C * Gm::KB, at, 16 * it, k), s);
              s = mma(KT::frag(kt + C * Gm::KB, at, 16 * u, k), q0, s);
            }
            if (k % 2 == 1) __builtin_amdgcn_sched_barrier(0);      // (registers: not all operands at once)
          }
          if (u == it) {
#pragma unroll
            for (int r = 0; r < 4; ++r) s[r] = 4 * l4 + r <= l15 ? s[r] : 0.f;
          }
        }
        quad_t q[NOPND];
        split_quad(s, q);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) *(quad_t*)(pt + (o * C + i) * Gm::PB + (16 * u + 4 * l4) * Gm::ES) = q[o];
      }
      __builtin_amdgcn_sched_barrier(0);
      // what the state in front of the chunk contributes: O^T = S^T Q'^T, rows of this wave's 16 columns
      f32x4 out[RT];
#pragma unroll
      for (int it = 0; it < RT; ++it) out[it] = zero4();
#pragma unroll
      for (int t = 0; t < NS; t += 2) {
        quad_t a0[NOPND], a1[NOPND];
        split_quad(S[t], a0);
        split_quad(S[t + 1], a1);
#pragma unroll
        for (int it = 0; it < RT; ++it) {
          const quad_t b0 = KT::quad(qt, at, 16 * it, t), b1 = KT::quad(qt, at, 16 * it, t + 1);
#pragma unroll
          for (int o = 0; o < NOPND; ++o) out[it] = mma_quads(a0[o], a1[o], b0, b1, out[it]);
          if constexpr (SPLIT) {
            const uint8_t* ql = qt + C * Gm::KB;
            out[it] = mma_quads(a0[0], a1[0], KT::quad(ql, at, 16 * it, t), KT::quad(ql, at, 16 * it, t + 1), out[it]);
          }
        }
        __builtin_amdgcn_sched_barrier(0);      // (registers: not all operands at once)
      }
      __syncthreads();
#pragma unroll
      for (int it = 0; it < RT; ++it) {
#pragma unroll
        for (int kk = 0; kk < RT / 2; ++kk) {
          if (2 * kk > it) continue;
#pragma unroll
          for (int o = 0; o < NOPND; ++o) {
            const uint8_t* pr = pt + (o * C + 16 * it + l15) * Gm::PB + (32 * kk + 4 * l4) * Gm::ES;
            const quad_t b0 = *(const quad_t*)pr, b1 = *(const quad_t*)(pr + 16 * Gm::ES);
            out[it] = mma_quads(vq[2 * kk], vq[2 * kk + 1], b0, b1, out[it]);
          }
        }
        const int i = 16 * it + l15;
        if (i < n)
          *(quad_t*)(p.o + (int64_t)(row0 + c0) * p.ldo + h * p.dv + dv0 + (uint32_t)(i * (int)p.ldo + 16 * wave + 4 * l4)) = to_quad(out[it]);
      }
    }
    if (c0 + n < count) fetch_low(c0 + n);
    // S <- e^(B_n) (S + K'^T V)
#pragma unroll
    for (int t = 0; t < NS; ++t) {
#pragma unroll
      for (int kk = 0; kk < RT / 2; ++kk)
#pragma unroll
        for (int o = 0; o < NOPND; ++o) {
          const uint8_t* k = kt + o * C * Gm::KB;
          S[t] = mma_quads(KT::column_quad(k, at, 32 * kk, t, l15, l4), KT::column_quad(k, at, 32 * kk + 16, t, l15, l4), vq[2 * kk],
                           vq[2 * kk + 1], S[t]);
        }
      S[t] *= *(const f32x4*)(tot + 16 * t + 4 * l4);
      if (t % 2 == 1) __builtin_amdgcn_sched_barrier(0);
    }
    __builtin_amdgcn_sched_barrier(0);
    if (c0 + n < count) fetch(c0 + n);                 // (here and not earlier: registers)
    // (no barrier: the next chunk writes B first, which nobody reads any more, and then waits)
  }
  if (!OUTPUT) {
    keep(idx);
    if (tid < DK && dv0 == 0) p.seg_decay[((int64_t)sg * p.H + h) * DK + tid] = total;
  } else if (idx == nseg - 1) {
    store_state(own, S);
  }
}

struct GlaDecodeArgs {
  const elem_t* x; int64_t ld;
  elem_t* o; int64_t ldo;
  float* state;
  const int *slot, *pos;                 // pos < 0: an empty place of the batch
  int64_t low_col;
  const elem_t* a2; const float* bias;
  int rp;
  float inv_tau, scale;
  int64_t g_col;
  const float* w;
  int n;
  float eps;
  int H;
};

template <int DK, int DV>
__global__ __launch_bounds__(4 * DV) void gla_decode_kernel(GlaDecodeArgs p) {
  constexpr int TH = 4 * DV, COLS = DV / 4, ROWS = DK / STATE_GROUPS;
  static_assert(TH == COLS * STATE_GROUPS, "layout");
  __shared__ float qs[DK], ks[DK], as[DK];
  __shared__ f32x4 red[STATE_GROUPS][COLS];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, col = tid % COLS, grp = tid / COLS;
  const int ps = p.pos[b];
  if (ps < 0) return;
  const elem_t* row = p.x + (int64_t)b * p.ld;
  float* S = p.state + ((int64_t)p.slot[b] * p.H + h) * DK * DV + 4 * col + (int64_t)grp * ROWS * DV;
  f32x4 s[ROWS];                         // requested before anything waits
#pragma unroll
  for (int i = 0; i < ROWS; ++i) s[i] = ps > 0 ? *(const f32x4*)(S + (int64_t)i * DV) : zero4();
  const f32x4 v = from_quad(*(const quad_t*)(row + (int64_t)2 * p.H * DK + (int64_t)h * DV + 4 * col));
  for (int d = tid; d < DK; d += TH) {
    const elem_t *a = p.a2 + (int64_t)(h * DK + d) * p.rp, *t = row + p.low_col;
    float z = p.bias[h * DK + d];
    for (int i = 0; i < p.rp; i += FR) {
      const frag_t u = *(const frag_t*)(a + i), w = *(const frag_t*)(t + i);
#pragma unroll
      for (int e = 0; e < FR; ++e) z += (float)u[e] * (float)w[e];
    }
    as[d] = __builtin_amdgcn_exp2f(log_decay(z, p.inv_tau));
    qs[d] = (float)row[(int64_t)h * DK + d] * p.scale;
    ks[d] = (float)row[(int64_t)(p.H + h) * DK + d];
  }
  __syncthreads();
  f32x4 acc = zero4();
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int d = grp * ROWS + i;
    s[i] = as[d] * s[i] + ks[d] * v;
    acc += qs[d] * s[i];
    *(f32x4*)(S + (int64_t)i * DV) = s[i];
  }
  const f32x4 y = over_groups<DV>(acc, red, grp, col);
  if (tid < COLS) {
    const HeadOut out{row + p.g_col + (int64_t)h * DV, p.w, p.n, p.eps};
    head_out<DV>(y, out, p.o + (int64_t)b * p.ldo + (int64_t)h * DV);
  }
}

template <int DK, int NWV>
static int launch(const GlaArgs& a, int segments, int multi, hipStream_t s) {
  constexpr size_t lds = GlaGeom<DK, NWV>::LDS;
  const dim3 grid(segments, a.H, a.dv / (16 * NWV)), block(64 * NWV);
  if (multi) {
    auto k = gla_prefill_kernel<DK, NWV, false>;
    if (allow_lds(k, lds)) return LM_EINVAL;
    hipLaunchKernelGGL(k, grid, block, lds, s, a);
  }
  auto k = gla_prefill_kernel<DK, NWV, true>;
  if (allow_lds(k, lds)) return LM_EINVAL;
  hipLaunchKernelGGL(k, grid, block, lds, s, a);
  return launch_status();
}

template <int DK>
static int plan(const GlaArgs& a, int segments, int multi, hipStream_t s) {
  if constexpr (SPLIT && DK <= 128) {
    if (a.dv % 128 == 0) return launch<DK, 8>(a, segments, multi, s);
  }
  return launch<DK, 4>(a, segments, multi, s);
}

}  // namespace lm

using namespace lm;

extern "C" int lm_gla_prefill(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* seg_state, float* seg_decay,
                              const int* seg, int segments, int multi, int64_t low_col, const void* a2, const float* bias, int rp,
                              float inv_tau, float scale, int H, int dk, int dv, void* stream) {
  if (segments <= 0 || H <= 0 || dv <= 0 || dv % 64 || (multi && (!seg_state || !seg_decay)) || ld > (1 << 24) || ldo > (1 << 24) || ld % FR || ldo % 4 || low_col % FR ||
      rp < 64 || rp % 64 || !(inv_tau > 0.f))
    return LM_EINVAL;
  GlaArgs a{(const elem_t*)x, ld, (elem_t*)o, ldo, state, seg_state, seg_decay, seg, low_col, (const elem_t*)a2, bias, rp, inv_tau, scale,
            H, dv};
  hipStream_t s = (hipStream_t)stream;
  if (dk == 64) return plan<64>(a, segments, multi, s);
  if (dk == 128) return plan<128>(a, segments, multi, s);
  if (dk == 256) return plan<256>(a, segments, multi, s);
  return LM_EINVAL;
}

extern "C" int lm_gla_decode(const void* x, int64_t ld, void* o, int64_t ldo, float* state, const int* slot, const int* pos,
                             int64_t low_col, const void* a2, const float* bias, int rp, float inv_tau, float scale, int64_t g_col,
                             const float* w, int n, float eps, int B, int H, int dk, int dv, void* stream) {
  if (B <= 0 || H <= 0 || n <= 0 || n > dv || ld % FR || ldo % 4 || low_col % FR || g_col % 4 || rp <= 0 || rp % FR || !(inv_tau > 0.f))
    return LM_EINVAL;
  GlaDecodeArgs a{(const elem_t*)x, ld, (elem_t*)o, ldo, state, slot, pos, low_col, (const elem_t*)a2, bias, rp, inv_tau, scale, g_col, w,
                  n, eps, H};
  hipStream_t s = (hipStream_t)stream;
#define LM_CASE(K, V)                                                                                        \
  if (dk == K && dv == V) {                                                                                  \
    hipLaunchKernelGGL((gla_decode_kernel<K, V>), dim3(B, H), dim3(4 * V), 0, s, a);                         \
    return launch_status();                                                                                  \
  }
  LM_CASE(64, 64) LM_CASE(64, 128) LM_CASE(64, 256) LM_CASE(128, 64) LM_CASE(128, 128) LM_CASE(128, 256)
  LM_CASE(256, 64) LM_CASE(256, 128) LM_CASE(256, 256)
#undef LM_CASE
  return LM_EINVAL;
}
