// Decayed linear attention  S_t = lam S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t  (per head; S f32 [dk][dv], one slot per sequence).
//
// Prompt portions, chunks of C tokens: with S the state before the chunk and i, j places in it (n of them)
//     o_i = lam^(i+1) S^T q_i + sum_{j <= i} lam^(i-j) (q_i . k_j) v_j          S' = lam^n S + sum_j lam^(n-1-j) k_j v_j^T
// A workgroup owns 64 or 128 value columns of one head and walks the chunks of one segment of a sequence; S stays in MFMA accumulators
// (16 columns per wave).  Its accumulator layout is the quad layout of S^T as an operand, so the state never passes through LDS.
// f32 factors (S, the decayed score matrix, the decayed values) enter the bf16 products as two bf16 operands each.
// Long portions are cut into segments that run in parallel: a first pass forms what each segment adds to the state, the second
// starts every segment from the decayed sum of those before it.
#include "lm_common.h"
#include "omniserve_lm.h"

namespace lm {

struct LinArgs {
  const elem_t* x; int64_t ld;         // row: q [H][dk], k [H][dk], v [H][dv] as projected
  elem_t* o; int64_t ldo;              // [tokens][H][dv]
  float* state;                        // [slots][H][dk][dv]
  float* seg_state;                    // [segments][H][dk][dv]
  const int* seg;                      // [segments][8]: first token, tokens, slot, 1 = starts from zero, index in its entry,
                                       //                segments of the entry, 0, 0
  const float* log2_decay;             // [H]
  int H, dv, seg_len, act;
};

template <int DK, int NWV>
struct LinGeom {
  static constexpr int TH = 64 * NWV, DVB = 16 * NWV;                  // threads, value columns of a workgroup
  static constexpr int C = SPLIT ? 64 : 32;                            // tokens per chunk
  static constexpr int KB = DK * (int)sizeof(elem_t), VB = DVB * (int)sizeof(elem_t);
  static constexpr int PB = C * (int)sizeof(elem_t) + 16;              // row of the score matrix
  static constexpr int Q0 = 0, K0 = C * KB, V0 = 2 * C * KB, P0 = V0 + C * VB, LDS = P0 + NOPND * C * PB;
  static constexpr int NQ = C * KB / (16 * TH), NV = C * VB / (16 * TH);         // 16-byte loads per thread
};

constexpr int linear_waves_per_simd(int dk, int waves) { return SPLIT && (dk <= 64 || waves == 8) ? 2 : 1; }      // what the registers allow

__device__ __forceinline__ frag_t activate(frag_t v, int act) {
  if (act == LM_ACT_SILU) {
#pragma unroll
    for (int e = 0; e < FR; ++e) v[e] = (elem_t)silu((float)v[e]);
  }
  return v;
}

template <int DK, int NWV, bool OUTPUT>
__global__ __launch_bounds__(64 * NWV, linear_waves_per_simd(DK, NWV)) void linear_prefill_kernel(LinArgs p) {
  typedef LinGeom<DK, NWV> Gm;
  typedef Tile<Gm::KB> KT;
  typedef Tile<Gm::VB> VT;
  constexpr int C = Gm::C, NS = DK / 16, NKF = DK / KSTEP, RT = C / 16;
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  uint8_t *qt = lds + Gm::Q0, *kt = lds + Gm::K0, *vt = lds + Gm::V0, *pt = lds + Gm::P0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int sg = blockIdx.x, h = blockIdx.y, dv0 = Gm::DVB * blockIdx.z;
  const int *sp = p.seg + 8 * sg;
  const int row0 = sp[0], count = sp[1], slot = sp[2], fresh = sp[3], idx = sp[4], nseg = sp[5];
  if (!OUTPUT && idx == nseg - 1) return;             // nothing follows the last segment
  const float ld = p.log2_decay[h];
  const int64_t st_stride = (int64_t)DK * p.dv;
  const int64_t sbase = (int64_t)4 * l4 * p.dv + dv0 + 16 * wave + l15;     // this lane's column, row 4 l4
  auto load_state = [&](const float* s, float f, f32x4 (&S)[NS]) {
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t][r] += f * s[sbase + (int64_t)(16 * t + r) * p.dv];
  };
  auto store_state = [&](float* s, const f32x4 (&S)[NS]) {
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) s[sbase + (int64_t)(16 * t + r) * p.dv] = S[t][r];
  };
  f32x4 S[NS];
#pragma unroll
  for (int t = 0; t < NS; ++t) S[t] = zero4();
  float* own = p.state + ((int64_t)slot * p.H + h) * st_stride;
  auto seg_at = [&](int i) { return p.seg_state + ((int64_t)(sg - idx + i) * p.H + h) * st_stride; };
  if (idx == 0) {
    if (OUTPUT && nseg > 1) {
      load_state(seg_at(nseg - 1), 1.0f, S);          // kept by the first pass: the last segment replaces the slot's state
    } else if (!fresh) {
      load_state(own, 1.0f, S);
    }
    if (!OUTPUT) store_state(seg_at(nseg - 1), S);
  } else if (OUTPUT) {
    for (int i = 0; i < idx; ++i) load_state(seg_at(i), power(ld, p.seg_len * (idx - 1 - i)), S);
  }

  const elem_t* src = p.x + (int64_t)row0 * p.ld;
  const int64_t qo = (int64_t)h * DK, ko = (int64_t)(p.H + h) * DK, vo = (int64_t)2 * p.H * DK + (int64_t)h * p.dv + dv0;
  frag_t rq[OUTPUT ? Gm::NQ : 1], rk[Gm::NQ], rv[Gm::NV];
  auto fetch = [&](int c0) {
#pragma unroll
    for (int i = 0; i < Gm::NQ; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / KT::NS, s = sl % KT::NS;
      const bool in = c0 + r < count;
      const elem_t* a = src + (int64_t)(in ? c0 + r : 0) * p.ld + s * FR;
      if constexpr (OUTPUT) rq[i] = in ? *(const frag_t*)(a + qo) : frag_t{};
      rk[i] = in ? *(const frag_t*)(a + ko) : frag_t{};
    }
#pragma unroll
    for (int i = 0; i < Gm::NV; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / VT::NS, s = sl % VT::NS;
      const bool in = c0 + r < count;
      rv[i] = in ? *(const frag_t*)(src + (int64_t)(c0 + r) * p.ld + vo + s * FR) : frag_t{};
    }
  };
  // decay factors of a whole chunk
  f32x4 wv[RT];                                        // of v_j in the new state
  float wo[RT];                                        // of the state in row i
#pragma unroll
  for (int u = 0; u < RT; ++u) {
#pragma unroll
    for (int r = 0; r < 4; ++r) wv[u][r] = power(ld, C - 1 - (16 * u + 4 * l4 + r));
    wo[u] = power(ld, 16 * u + l15 + 1);
  }
  const float wc = power(ld, C), ld1 = power(ld, 1), ld2 = ld1 * ld1, ld3 = ld2 * ld1;
  fetch(0);
  for (int c0 = 0; c0 < count; c0 += C) {
    const int n = min(C, count - c0);
#pragma unroll
    for (int i = 0; i < Gm::NQ; ++i) {
      const int sl = Gm::TH * i + tid, off = KT::slot(sl / KT::NS, sl % KT::NS);
      if constexpr (OUTPUT) *(frag_t*)(qt + off) = activate(rq[i], p.act);
      *(frag_t*)(kt + off) = activate(rk[i], p.act);
    }
#pragma unroll
    for (int i = 0; i < Gm::NV; ++i) {
      const int sl = Gm::TH * i + tid;
      *(frag_t*)(vt + VT::slot(sl / VT::NS, sl % VT::NS)) = activate(rv[i], p.act);
    }
    __syncthreads();
    if (c0 + C < count) fetch(c0 + C);
    quad_t vq[RT][1];                                  // V, column l15 of this wave, all tokens of the chunk
#pragma unroll
    for (int u = 0; u < RT; ++u) vq[u][0] = VT::column_quad(vt, 16 * u, wave, l15, l4);
    if constexpr (OUTPUT) {
      // decayed scores (transposed product: column = row i of the score matrix); blocks (row it, key u) of the lower triangle
      // go round the waves.  The block right of an even diagonal block is read behind: zeros.
      constexpr int BLOCKS = RT * RT;
#pragma unroll
      for (int bi = 0; bi < (BLOCKS + NWV - 1) / NWV; ++bi) {
        const int it = wave % RT, u = bi * (NWV / RT > 0 ? NWV / RT : 1) + wave / RT;
        if (it >= RT || u >= RT || u > (it | 1)) continue;
        const int i = 16 * it + l15;
        f32x4 s = zero4();
        if (u <= it) {
#pragma unroll
          for (int k = 0; k < NKF; ++k) s = mma(KT::frag(kt, 16 * u + l15, 4 * k + l4), KT::frag(qt, i, 4 * k + l4), s);
          const int d0 = i - (16 * u + 4 * l4);       // distance of the lane's first key
          if (u < it) {
            const float f = power(ld, d0 - 3);
            s *= (f32x4){f * ld3, f * ld2, f * ld1, f};
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) s[r] = d0 >= r ? s[r] * power(ld, d0 - r) : 0.f;
          }
        }
        quad_t q[NOPND];
        split_quad(s, q);
#pragma unroll
        for (int o = 0; o < NOPND; ++o)
          *(quad_t*)(pt + (o * C + i) * Gm::PB + (16 * u + 4 * l4) * (int)sizeof(elem_t)) = q[o];
      }
      // what the state in front of the chunk contributes: O^T = S^T Q^T, rows of this wave's 16 columns
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
          const quad_t b0 = KT::quad(qt, 16 * it + l15, t, l4), b1 = KT::quad(qt, 16 * it + l15, t + 1, l4);
#pragma unroll
          for (int o = 0; o < NOPND; ++o) out[it] = mma_quads(a0[o], a1[o], b0, b1, out[it]);
        }
      }
#pragma unroll
      for (int it = 0; it < RT; ++it) out[it] *= wo[it];
      __syncthreads();
#pragma unroll
      for (int it = 0; it < RT; ++it) {
#pragma unroll
        for (int kk = 0; kk < RT / 2; ++kk) {
          if (2 * kk > it) continue;
#pragma unroll
          for (int o = 0; o < NOPND; ++o) {
            const uint8_t* pr = pt + (o * C + 16 * it + l15) * Gm::PB + (32 * kk + 4 * l4) * (int)sizeof(elem_t);
            const quad_t b0 = *(const quad_t*)pr, b1 = *(const quad_t*)(pr + 16 * (int)sizeof(elem_t));
            out[it] = mma_quads(vq[2 * kk][0], vq[2 * kk + 1][0], b0, b1, out[it]);
          }
        }
        const int i = 16 * it + l15;
        if (i < n)
          *(quad_t*)(p.o + (int64_t)(row0 + c0 + i) * p.ldo + (int64_t)h * p.dv + dv0 + 16 * wave + 4 * l4) = to_quad(out[it]);
      }
    }
    // S <- lam^n S + K^T (lam^(n-1-j) v_j)
    const float fn = n == C ? wc : power(ld, n);
#pragma unroll
    for (int t = 0; t < NS; ++t) S[t] *= fn;
#pragma unroll
    for (int kk = 0; kk < RT / 2; ++kk) {
      quad_t b0[NOPND], b1[NOPND];
      f32x4 x0 = from_quad(vq[2 * kk][0]), x1 = from_quad(vq[2 * kk + 1][0]);
      if (n == C) {
        x0 *= wv[2 * kk];
        x1 *= wv[2 * kk + 1];
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = 32 * kk + 4 * l4 + r;          // (places from n on hold zeros)
          x0[r] *= power(ld, max(n - 1 - j, 0));
          x1[r] *= power(ld, max(n - 1 - j - 16, 0));
        }
      }
      split_quad(x0, b0);
      split_quad(x1, b1);
#pragma unroll
      for (int t = 0; t < NS; ++t) {
        const quad_t a0 = KT::column_quad(kt, 32 * kk, t, l15, l4), a1 = KT::column_quad(kt, 32 * kk + 16, t, l15, l4);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) S[t] = mma_quads(a0, a1, b0[o], b1[o], S[t]);
      }
    }
    __syncthreads();
  }
  if (!OUTPUT) store_state(seg_at(idx), S);
  else if (idx == nseg - 1) store_state(own, S);
}

// One token per sequence.  A workgroup owns one head: thread = 4 value columns x dk / GROUPS rows; sums over the row groups
// meet in LDS.
__global__ __launch_bounds__(256) void linear_decode_kernel(const elem_t* x, int64_t ldx, elem_t* o, int64_t ldo, float* state,
                                                            const int* slot, const int* pos, const float* log2_decay, int H, int dk,
                                                            int dv, int act) {
  __shared__ float qk[2][256];
  __shared__ f32x4 red[256];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int ps = pos[b];
  if (ps < 0) return;
  const elem_t* row = x + (int64_t)b * ldx;
  const int cols = dv / 4, groups = 256 / cols, col = tid % cols, grp = tid / cols, per = dk / groups;
  float* S = state + ((int64_t)slot[b] * H + h) * dk * dv + 4 * col + (int64_t)grp * per * dv;
  auto f = [act](float v) { return act == LM_ACT_SILU ? (float)(elem_t)silu(v) : v; };
  f32x4 s[8];                                           // the first rows are requested before anything waits
#pragma unroll
  for (int i = 0; i < 8; ++i) s[i] = ps > 0 && i < per ? *(const f32x4*)(S + (int64_t)i * dv) : zero4();
  if (tid < dk) {
    qk[0][tid] = f((float)row[(int64_t)h * dk + tid]);
    qk[1][tid] = f((float)row[(int64_t)(H + h) * dk + tid]);
  }
  f32x4 v = from_quad(*(const quad_t*)(row + (int64_t)2 * H * dk + (int64_t)h * dv + 4 * col));
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = f(v[e]);
  const float lam = power(log2_decay[h], 1);
  __syncthreads();
  f32x4 acc = zero4();
  for (int i0 = 0; i0 < per; i0 += 8) {
    f32x4 nx[8];
    if (i0 + 8 < per) {
#pragma unroll
      for (int i = 0; i < 8; ++i) nx[i] = ps > 0 && i0 + 8 + i < per ? *(const f32x4*)(S + (int64_t)(i0 + 8 + i) * dv) : zero4();
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if (i0 + i < per) {
        const int d = grp * per + i0 + i;
        s[i] = lam * s[i] + qk[1][d] * v;
        acc += qk[0][d] * s[i];
        *(f32x4*)(S + (int64_t)(i0 + i) * dv) = s[i];
      }
    }
    if (i0 + 8 < per) {
#pragma unroll
      for (int i = 0; i < 8; ++i) s[i] = nx[i];
    }
  }
  red[tid] = acc;
  __syncthreads();
  if (tid < cols) {
    for (int g = 1; g < groups; ++g) acc += red[g * cols + tid];
    *(quad_t*)(o + (int64_t)b * ldo + (int64_t)h * dv + 4 * tid) = to_quad(acc);
  }
}

template <int DK, int NWV>
static int launch(const LinArgs& a, int segments, int multi, hipStream_t s) {
  constexpr size_t lds = LinGeom<DK, NWV>::LDS;
  const dim3 grid(segments, a.H, a.dv / (16 * NWV)), block(64 * NWV);
  if (multi) {
    auto k = linear_prefill_kernel<DK, NWV, false>;
    if (allow_lds(k, lds)) return LM_EINVAL;
    hipLaunchKernelGGL(k, grid, block, lds, s, a);
  }
  auto k = linear_prefill_kernel<DK, NWV, true>;
  if (allow_lds(k, lds)) return LM_EINVAL;
  hipLaunchKernelGGL(k, grid, block, lds, s, a);
  return launch_status();
}

// 128 value columns share one staging of q and k where the registers allow
template <int DK>
static int plan(const LinArgs& a, int segments, int multi, hipStream_t s) {
  if constexpr (SPLIT && DK <= 128) {
    if (a.dv % 128 == 0) return launch<DK, 8>(a, segments, multi, s);
  }
  return launch<DK, 4>(a, segments, multi, s);
}

}  // namespace lm

using namespace lm;

extern "C" int lm_linear_prefill(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* seg_state, const int* seg,
                                 int segments, int seg_len, int multi, const float* log2_decay, int H, int dk, int dv, int act,
                                 void* stream) {
  if (segments <= 0 || H <= 0 || dv % 64 || seg_len % 64 || seg_len <= 0 || (multi && !seg_state) || ld % FR || ldo % 4) return LM_EINVAL;
  LinArgs a{(const elem_t*)x, ld, (elem_t*)o, ldo, state, seg_state, seg, log2_decay, H, dv, seg_len, act};
  hipStream_t s = (hipStream_t)stream;
  if (dk == 64) return plan<64>(a, segments, multi, s);
  if (dk == 128) return plan<128>(a, segments, multi, s);
  if (dk == 256) return plan<256>(a, segments, multi, s);
  return LM_EINVAL;
}

extern "C" int lm_linear_decode(const void* x, int64_t ld, void* o, int64_t ldo, float* state, const int* slot, const int* pos,
                                const float* log2_decay, int B, int H, int dk, int dv, int act, void* stream) {
  if (B <= 0 || H <= 0 || (dk != 64 && dk != 128 && dk != 256) || (dv != 64 && dv != 128 && dv != 256) || ld % 4 || ldo % 4)
    return LM_EINVAL;
  hipLaunchKernelGGL(linear_decode_kernel, dim3(B, H), dim3(256), 0, (hipStream_t)stream, (const elem_t*)x, ld, (elem_t*)o, ldo, state,
                     slot, pos, log2_decay, H, dk, dv, act);
  return launch_status();
}
