// Gated delta rule  S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q   (per head; S f32 [dk][dv], one slot per sequence),
// q, k, v behind a short causal convolution and silu, q and k unit vectors, q times scale; g and beta one number per head and token.
//
// Prompt portions, chunks of C tokens.  With q~, k~ the convolved vectors, rq, rk the factors that make them unit vectors, G_i the
// running sum of log g within the chunk and S the state in front of it, the written vectors u solve a triangular system:
//     (I + A) U = diag(beta) (V - diag(e^G rk) K~ S),      A_ij = beta_i e^(G_i - G_j) rk_i rk_j (k~_i . k~_j), j < i
//     o_i = e^(G_i) rq_i S^T q~_i + sum_{j <= i} P_ij u_j,    P_ij = e^(G_i - G_j) rq_i rk_j (q~_i . k~_j)
//     S'  = e^(G_n) S + sum_j (e^(G_n - G_j) rk_j) k~_j u_j^T
// All exponents are sums of log g <= 0.  Three launches:
//   conv      convolution + silu of every channel, the factors rq and rk (parallel over tokens)
//   chunk     one wave per (chunk, head): A and P by MFMA, T = (I + A)^-1 diag(beta) by forward substitution, one column per lane;
//             the last inputs of a portion go to the ring of its slot
//   prefill   one workgroup per (segment, head, 64 value columns) walks the chunks: R = V - diag(e^G rk) K~ S, U = T R, the outputs
//             and the next state.  S stays in MFMA accumulators; every result tile is the next product's operand as it lies.
// Long portions are cut into segments that run in parallel.  A segment takes a state S to M S + C: a first pass forms C (the segment
// from a zero state) and, as dk more columns, M (the segment without values, from the identity); `chain` turns the C into the states
// behind the segments, from which the second pass starts.
// f32 factors (S, R, U, T, P) enter the bf16 products as two bf16 operands each; of two such factors the product of the two low
// parts is dropped.
#include "lm_state.h"
#include "omniserve_lm.h"

namespace lm {

constexpr int DC = SPLIT ? 64 : 32;                       // tokens per chunk
constexpr int64_t MATS = (int64_t)2 * NOPND * DC * DC;    // elements of T and P of one chunk and head

struct DeltaArgs {
  const elem_t* x; int64_t ld;           // row: q [G][dk], k [G][dk], v [H][dv] as projected; from ab_col on a [H], b [H]
  elem_t* o; int64_t ldo;                // [tokens][H][dv]
  float* state;                          // [slots][H][dk][dv]
  float* ring;                           // [slots][taps][channels]: the input of position p in row p % taps
  const int* portion;                    // [.][8]: first token, tokens, slot, 1 = starts from zero, first chunk, chunks, position, 0
  const int* chunks;                     // [n_chunks]: its portion
  const int* seg;                        // [segments][8]: first token, tokens, slot, 1 = starts from zero, index in its portion,
                                         //                segments of the portion, first chunk, 0
  float* seg_state;                      // [segments][H]: C [dk * dv] as the accumulators hold it, M [dk][dk]
  const float* conv_w; int taps;         // [taps][channels], the last row meets the current token
  float qk_eps, scale;
  int64_t ab_col;
  const float *a_log, *dt_bias;          // [H]
  elem_t* y;                             // [tokens][channels]: convolved
  float* norms;                          // [tokens][2 G]: rq, rk
  elem_t* mats;                          // [n_chunks][H][2][NOPND][DC][DC]: T, P
  float* vecs;                           // [n_chunks][H][4][DC]: e^G rk, e^G rq, e^(G_n - G) rk, e^(G_n)
  int H, G, dk, dv;
};

// ---- convolution, silu, unit-vector factors; 256 threads x FR channels, CONV_TOKENS tokens of a chunk ----
constexpr int CONV_TOKENS = 16;

// TAPS > 0: taps known, weights and the inputs on their way through stay in registers; 0: any number
template <int TAPS>
__global__ __launch_bounds__(256) void delta_conv_kernel(DeltaArgs p) {
  const int channels = 2 * p.G * p.dk + p.H * p.dv, c = (blockIdx.y * 256 + threadIdx.x) * FR;
  const int ck = blockIdx.x / (DC / CONV_TOKENS), part = blockIdx.x % (DC / CONV_TOKENS);
  const int* pp = p.portion + 8 * p.chunks[ck];
  const int first = pp[0], count = pp[1], slot = pp[2], pos0 = pp[6];
  const int t0 = (ck - pp[4]) * DC + part * CONV_TOKENS;       // within the portion
  if (c >= channels) return;
  const int qk = p.G * p.dk, lanes = p.dk / FR;
  auto input = [&](int t) -> frag_t {                           // of place t, which may lie before the portion
    if (t >= 0) return *(const frag_t*)(p.x + (int64_t)(first + t) * p.ld + c);
    frag_t v = {};
    if (pos0 + t >= 0) {
      const float* r = p.ring + ((int64_t)slot * p.taps + (pos0 + t) % p.taps) * channels + c;
#pragma unroll
      for (int e = 0; e < FR; ++e) v[e] = (elem_t)r[e];         // (an element's value)
    }
    return v;
  };
  auto finish = [&](int t, const float (&s)[FR]) {
    frag_t y;
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < FR; ++e) {
      y[e] = (elem_t)silu(s[e]);
      ss += (float)y[e] * (float)y[e];
    }
    *(frag_t*)(p.y + (int64_t)(first + t) * channels + c) = y;
    if (c < 2 * qk) {                                           // whole groups of lanes: heads are multiples of 64 channels
      for (int m = lanes >> 1; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
      if (c % p.dk == 0)
        p.norms[(int64_t)(first + t) * 2 * p.G + c / p.dk] = (c < qk ? p.scale : 1.0f) / sqrtf(ss + p.qk_eps);
    }
  };
  const int t1 = min(t0 + CONV_TOKENS, count);
  if constexpr (TAPS > 0) {
    if (t0 >= t1) return;
    constexpr int B = 4;                                        // inputs requested together
    float w[TAPS][FR];
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int e = 0; e < FR; ++e) w[j][e] = p.conv_w[(int64_t)j * channels + c + e];
    frag_t in[TAPS - 1 + B];
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) in[j] = input(t0 - (TAPS - 1) + j);
    for (int t = t0; t < t1; t += B) {
#pragma unroll
      for (int b = 0; b < B; ++b) in[TAPS - 1 + b] = input(min(t + b, t1 - 1));
#pragma unroll
      for (int b = 0; b < B; ++b) {
        if (t + b >= t1) break;
        float s[FR];
#pragma unroll
        for (int e = 0; e < FR; ++e) s[e] = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
#pragma unroll
          for (int e = 0; e < FR; ++e) s[e] += w[j][e] * (float)in[b + j][e];
        finish(t + b, s);
      }
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) in[j] = in[B + j];
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      float s[FR];
#pragma unroll
      for (int e = 0; e < FR; ++e) s[e] = 0.f;
      for (int j = 0; j < p.taps; ++j) {
        const frag_t v = input(t - (p.taps - 1) + j);
#pragma unroll
        for (int e = 0; e < FR; ++e) s[e] += p.conv_w[(int64_t)j * channels + c + e] * (float)v[e];
      }
      finish(t, s);
    }
  }
}

// ---- the chunk's matrices ----
template <int DK>
__global__ __launch_bounds__(64) void delta_chunk_kernel(DeltaArgs p) {
  constexpr int RT = DC / 16, NKF = DK / KSTEP, AP = DC + 4;
  __shared__ __attribute__((aligned(16))) float A[DC][AP];
  __shared__ float Gs[DC], be[DC], rqs[DC], rks[DC];
  const int lane = threadIdx.x, l15 = lane & 15, l4 = lane >> 4;
  const int ck = blockIdx.y, h = blockIdx.x, g = h / (p.H / p.G);
  const int* pp = p.portion + 8 * p.chunks[ck];
  const int first = pp[0], count = pp[1], slot = pp[2], nch = pp[5], pos0 = pp[6], index = ck - pp[4];
  const int t0 = index * DC, n = min(DC, count - t0);
  const int channels = 2 * p.G * p.dk + p.H * p.dv;
  float beta = 0.f;
  {
    float lg = 0.f, rq = 0.f, rk = 0.f;
    if (lane < n) {
      const int64_t t = first + t0 + lane;
      const elem_t* ab = p.x + t * p.ld + p.ab_col;
      lg = -__expf(p.a_log[h]) * softplus((float)ab[h] + p.dt_bias[h]) * LOG2E;
      beta = sigmoid((float)ab[p.H + h]);
      rq = p.norms[t * 2 * p.G + g];
      rk = p.norms[t * 2 * p.G + p.G + g];
    }
    float G = lg;
#pragma unroll
    for (int m = 1; m < 64; m <<= 1) {
      const float v = __shfl_up(G, m, 64);
      G += lane >= m ? v : 0.f;
    }
    const float all = __shfl(G, 63, 64);
    if (lane < DC) {
      Gs[lane] = G; be[lane] = beta; rqs[lane] = rq; rks[lane] = rk;
      float* v = p.vecs + ((int64_t)ck * p.H + h) * 4 * DC + lane;
      const float e = __builtin_amdgcn_exp2f(G);
      v[0] = e * rk;
      v[DC] = e * rq;
      v[2 * DC] = __builtin_amdgcn_exp2f(all - G) * rk;
      v[3 * DC] = __builtin_amdgcn_exp2f(all);
    }
  }
  __syncthreads();
  elem_t* mt = p.mats + ((int64_t)ck * p.H + h) * MATS;
  elem_t* mp = mt + NOPND * DC * DC;
  const elem_t* yq = p.y + (int64_t)(first + t0) * channels + (int64_t)g * DK;
  const elem_t* yk = yq + (int64_t)p.G * DK;
  frag_t kf[RT][NKF], qf[2][NKF];                // all keys, the queries one block ahead
  auto row_at = [&](int blk) { return (uint32_t)(min(16 * blk + l15, n - 1) * channels + FR * l4); };
#pragma unroll
  for (int u = 0; u < RT; ++u)
#pragma unroll
    for (int s = 0; s < NKF; ++s) kf[u][s] = *(const frag_t*)(yk + (row_at(u) + s * KSTEP));
#pragma unroll
  for (int s = 0; s < NKF; ++s) qf[0][s] = *(const frag_t*)(yq + (row_at(0) + s * KSTEP));
#pragma unroll
  for (int it = 0; it < RT; ++it) {              // rows i of block it against keys j of blocks u <= it (and the zeros beside them)
    if (it + 1 < RT) {
#pragma unroll
      for (int s = 0; s < NKF; ++s) qf[(it + 1) & 1][s] = *(const frag_t*)(yq + (row_at(it + 1) + s * KSTEP));
    }
#pragma unroll
    for (int u = 0; u < RT; ++u) {
      const int i = 16 * it + l15, j = 16 * u + 4 * l4;
      f32x4 kk = zero4(), qk = zero4();
      if (u <= it) {
#pragma unroll
        for (int s = 0; s < NKF; ++s) {
          kk = mma(kf[u][s], kf[it][s], kk);
          qk = mma(kf[u][s], qf[it & 1][s], qk);
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float d = j + r <= i ? __builtin_amdgcn_exp2f(Gs[i] - Gs[j + r]) * rks[j + r] : 0.f;
        kk[r] = j + r < i ? kk[r] * d * rks[i] * be[i] : 0.f;
        qk[r] *= d * rqs[i];
      }
      *(f32x4*)&A[i][j] = kk;
      quad_t q[NOPND];
      split_quad(qk, q);
#pragma unroll
      for (int o = 0; o < NOPND; ++o) *(quad_t*)(mp + (int64_t)o * DC * DC + i * DC + j) = q[o];
    }
  }
  __syncthreads();
  // column `lane` of (I + A)^-1, times beta of its token
  float x[DC];
#pragma unroll
  for (int i = 0; i < DC; ++i) {
    float s = i == lane ? 1.0f : 0.0f;
#pragma unroll
    for (int j = 0; j + 4 <= (i + 3) / 4 * 4; j += 4) {
      const f32x4 a = *(const f32x4*)&A[i][j];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (j + r < i) s -= a[r] * x[j + r];
    }
    x[i] = s;
  }
  if (lane < DC) {
#pragma unroll
    for (int i = 0; i < DC; ++i) {
      const float v = x[i] * beta;
      const elem_t hi = (elem_t)v;
      mt[i * DC + lane] = hi;
      if constexpr (SPLIT) mt[DC * DC + i * DC + lane] = (elem_t)(v - (float)hi);
    }
  }
  // the portion's last inputs
  if (index == nch - 1) {
    const int heads = p.H / p.G;
    for (int j = 0; j < min(p.taps - 1, count); ++j) {
      const elem_t* s = p.x + (int64_t)(first + count - 1 - j) * p.ld;
      float* d = p.ring + ((int64_t)slot * p.taps + (pos0 + count - 1 - j) % p.taps) * channels;
      for (int c = lane; c < p.dv; c += 64) d[2 * p.G * DK + h * p.dv + c] = (float)s[2 * p.G * DK + h * p.dv + c];
      if (h % heads == 0)
        for (int c = lane; c < DK; c += 64) {
          d[g * DK + c] = (float)s[g * DK + c];
          d[(p.G + g) * DK + c] = (float)s[(p.G + g) * DK + c];
        }
    }
  }
}

// ---- the recurrence over a portion's chunks ----
template <int DK, bool OUTPUT>
struct DeltaGeom {
  static constexpr int NWV = 4, TH = 256, DVB = 64, ES = (int)sizeof(elem_t);
  static constexpr int KB = DK * ES, VB = DVB * ES, PB = DC * ES + 16;
  static constexpr int Q0 = 0, K0 = OUTPUT ? DC * KB : 0, V0 = K0 + DC * KB, M0 = V0 + DC * VB, S0 = M0 + (OUTPUT ? 2 : 1) * NOPND * DC * PB,
                       LDS = S0 + 4 * DC * 4;
  static constexpr int NQ = DC * KB / (16 * TH), NV = DC * VB / (16 * TH);
  static constexpr int MR = DC * ES / 16, NM = (OUTPUT ? 2 : 1) * NOPND * DC * MR / TH;      // 16-byte pieces of a matrix row, per thread
  static_assert(NQ >= 1 && NV >= 1 && NM >= 1 && NOPND * DC * MR % TH == 0, "loads");
};

template <int DK, bool OUTPUT>
__global__ __launch_bounds__(256, !SPLIT || DK > 128 ? 1 : OUTPUT ? 2 : 3) void delta_prefill_kernel(DeltaArgs p) {
  typedef DeltaGeom<DK, OUTPUT> Gm;
  typedef Tile<Gm::KB> KT;
  typedef Tile<Gm::VB> VT;
  constexpr int NS = DK / 16, RT = DC / 16, MP = NOPND * DC * Gm::PB;      // MP: bytes of one matrix
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  uint8_t *qt = lds + Gm::Q0, *kt = lds + Gm::K0, *vt = lds + Gm::V0, *mt = lds + Gm::M0;
  float* vec = (float*)(lds + Gm::S0);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int sg = blockIdx.x;
  const int* sp = p.seg + 8 * sg;
  const int row0 = sp[0], count = sp[1], slot = sp[2], fresh = sp[3], idx = sp[4], nseg = sp[5], ck0 = sp[6], nch = (count + DC - 1) / DC;
  const int h = blockIdx.y, g = h / (p.H / p.G);
  const bool matrix = !OUTPUT && (int)blockIdx.z >= p.dv / Gm::DVB;      // columns of M
  const int dv0 = Gm::DVB * (matrix ? blockIdx.z - p.dv / Gm::DVB : blockIdx.z);
  if (!OUTPUT && (idx == nseg - 1 || (matrix && idx == 0))) return;      // nothing follows; nothing is in front
  const int channels = 2 * p.G * DK + p.H * p.dv;
  float* own = p.state + ((int64_t)slot * p.H + h) * DK * p.dv;
  const uint32_t sbase = 4 * l4 * p.dv + dv0 + 16 * wave + l15;         // this lane's column, row 4 l4
  f32x4 S[NS];
#pragma unroll
  for (int t = 0; t < NS; ++t) S[t] = zero4();
  auto seg_at = [&](int i) { return p.seg_state + ((int64_t)(sg - idx + i) * p.H + h) * DK * (p.dv + DK); };
  auto seg_cols = [&](int i) { return (f32x4*)(seg_at(i) + (dv0 + 16 * wave) * DK) + lane; };      // C, this wave's columns
  auto keep = [&](int i) {
    f32x4* s = seg_cols(i);
#pragma unroll
    for (int t = 0; t < NS; ++t) s[64 * t] = S[t];
  };
  auto recall = [&](int i) {
    const f32x4* s = seg_cols(i);
#pragma unroll
    for (int t = 0; t < NS; ++t) S[t] = s[64 * t];
  };
  if (matrix) {
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t][r] = 16 * t + 4 * l4 + r == dv0 + 16 * wave + l15 ? 1.0f : 0.0f;
  } else if (idx == 0) {
    if (OUTPUT && nseg > 1) {
      recall(nseg - 1);                   // kept by the first pass: the last segment replaces the slot's state
    } else if (!fresh) {
#pragma unroll
      for (int t = 0; t < NS; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[t][r] = own[sbase + (uint32_t)((16 * t + r) * p.dv)];
    }
    if (!OUTPUT) keep(nseg - 1);
  } else if (OUTPUT) {
    recall(idx - 1);                      // delta_chain_kernel has left the state behind every segment there
  }

  const elem_t* src = p.y + (int64_t)row0 * channels;
  const int qo = g * DK, ko = (p.G + g) * DK, vo = 2 * p.G * DK + h * p.dv + dv0;
  frag_t rq[OUTPUT ? Gm::NQ : 1], rk[Gm::NQ], rv[Gm::NV], rm[Gm::NM];      // (of the matrices T comes first)
  float rvec = 0.f;
  auto fetch = [&](int ck) {              // addresses: a base all lanes share, 32-bit offsets
    const elem_t* base = src + (int64_t)ck * DC * channels;
    const int last = count - 1 - ck * DC;
#pragma unroll
    for (int i = 0; i < Gm::NQ; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / KT::NS, s = sl % KT::NS;
      const uint32_t off = min(r, last) * channels + s * FR;
      if constexpr (OUTPUT) rq[i] = *(const frag_t*)(base + qo + off);
      rk[i] = *(const frag_t*)(base + ko + off);
    }
#pragma unroll
    for (int i = 0; i < Gm::NV; ++i) {
      const int sl = Gm::TH * i + tid, r = sl / VT::NS, s = sl % VT::NS;
      rv[i] = matrix ? frag_t{} : *(const frag_t*)(base + vo + (uint32_t)(min(r, last) * channels + s * FR));
    }
    const int64_t block = (int64_t)(ck0 + ck) * p.H + h;
#pragma unroll
    for (int i = 0; i < Gm::NM; ++i) rm[i] = *(const frag_t*)(p.mats + block * MATS + (uint32_t)((Gm::TH * i + tid) * FR));
    if (tid < 4 * DC) rvec = (p.vecs + block * 4 * DC)[(uint32_t)tid];
  };
  static_assert(4 * DC <= Gm::TH, "one factor per thread");
  fetch(0);
  typename KT::Offsets at(l15, l4);
  for (int ck = 0; ck < nch; ++ck) {
    const int n = min(DC, count - ck * DC);
    at.forget();
#pragma unroll
    for (int i = 0; i < Gm::NQ; ++i) {
      const int sl = Gm::TH * i + tid, off = KT::slot(sl / KT::NS, sl % KT::NS);
      if constexpr (OUTPUT) *(frag_t*)(qt + off) = rq[i];
      *(frag_t*)(kt + off) = rk[i];
    }
#pragma unroll
    for (int i = 0; i < Gm::NV; ++i) {
      const int sl = Gm::TH * i + tid;
      *(frag_t*)(vt + VT::slot(sl / VT::NS, sl % VT::NS)) = rv[i];
    }
#pragma unroll
    for (int i = 0; i < Gm::NM; ++i) {
      const int sl = Gm::TH * i + tid;
      *(frag_t*)(mt + (sl / Gm::MR) * Gm::PB + (sl % Gm::MR) * 16) = rm[i];
    }
    if (tid < 4 * DC) vec[tid] = rvec;
    __syncthreads();
    if (ck + 1 < nch) fetch(ck + 1);
    // R = V - diag(e^G rk) K~ S: rows tokens, column l15 of this wave; O^T = S^T Q~^T
    f32x4 R[RT], out[RT];
#pragma unroll
    for (int u = 0; u < RT; ++u) R[u] = out[u] = zero4();
#pragma unroll
    for (int t = 0; t < NS; t += 2) {
      quad_t s0[NOPND], s1[NOPND];
      split_quad(S[t], s0);
      split_quad(S[t + 1], s1);
#pragma unroll
      for (int u = 0; u < RT; ++u) {
        const quad_t k0 = KT::quad(kt, at, 16 * u, t), k1 = KT::quad(kt, at, 16 * u, t + 1);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) R[u] = mma_quads(k0, k1, s0[o], s1[o], R[u]);
        if constexpr (OUTPUT) {
          const quad_t q0 = KT::quad(qt, at, 16 * u, t), q1 = KT::quad(qt, at, 16 * u, t + 1);
#pragma unroll
          for (int o = 0; o < NOPND; ++o) out[u] = mma_quads(s0[o], s1[o], q0, q1, out[u]);
        }
      }
    }
    quad_t rs[RT][NOPND];
#pragma unroll
    for (int u = 0; u < RT; ++u) {
      const f32x4 wk = *(const f32x4*)(vec + 16 * u + 4 * l4);
      split_quad(from_quad(VT::column_quad(vt, 16 * u, wave, l15, l4)) - wk * R[u], rs[u]);
      out[u] *= vec[DC + 16 * u + l15];
    }
    // U = T R, rows tokens
    auto mat = [&](int m, int o, int row, int blk) -> quad_t {
      return *(const quad_t*)(mt + m * MP + (o * DC + row) * Gm::PB + (16 * blk + 4 * l4) * Gm::ES);
    };
    f32x4 U[RT];
#pragma unroll
    for (int it = 0; it < RT; ++it) {
      U[it] = zero4();
#pragma unroll
      for (int kk = 0; kk < RT / 2; ++kk) {
        if (2 * kk > it) continue;
        const quad_t a0 = mat(0, 0, 16 * it + l15, 2 * kk), a1 = mat(0, 0, 16 * it + l15, 2 * kk + 1);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) U[it] = mma_quads(a0, a1, rs[2 * kk][o], rs[2 * kk + 1][o], U[it]);
        if constexpr (SPLIT)
          U[it] = mma_quads(mat(0, 1, 16 * it + l15, 2 * kk), mat(0, 1, 16 * it + l15, 2 * kk + 1), rs[2 * kk][0], rs[2 * kk + 1][0], U[it]);
      }
    }
    // O^T += U^T P^T
    quad_t us[RT][NOPND];
    if constexpr (OUTPUT) {
#pragma unroll
      for (int u = 0; u < RT; ++u) split_quad(U[u], us[u]);
    }
#pragma unroll
    for (int it = 0; it < (OUTPUT ? RT : 0); ++it) {
#pragma unroll
      for (int kk = 0; kk < RT / 2; ++kk) {
        if (2 * kk > it) continue;
        const quad_t b0 = mat(1, 0, 16 * it + l15, 2 * kk), b1 = mat(1, 0, 16 * it + l15, 2 * kk + 1);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) out[it] = mma_quads(us[2 * kk][o], us[2 * kk + 1][o], b0, b1, out[it]);
        if constexpr (SPLIT)
          out[it] = mma_quads(us[2 * kk][0], us[2 * kk + 1][0], mat(1, 1, 16 * it + l15, 2 * kk), mat(1, 1, 16 * it + l15, 2 * kk + 1), out[it]);
      }
      const int i = 16 * it + l15;
      if (i < n)
        *(quad_t*)(p.o + (int64_t)(row0 + ck * DC) * p.ldo + h * p.dv + dv0 + (uint32_t)(i * (int)p.ldo + 16 * wave + 4 * l4)) = to_quad(out[it]);
    }
    // S <- e^(G_n) S + K~^T diag(e^(G_n - G) rk) U
    const float f = vec[3 * DC];
#pragma unroll
    for (int t = 0; t < NS; ++t) S[t] *= f;
#pragma unroll
    for (int u = 0; u < RT; ++u) split_quad(U[u] * *(const f32x4*)(vec + 2 * DC + 16 * u + 4 * l4), us[u]);
#pragma unroll
    for (int kk = 0; kk < RT / 2; ++kk)
#pragma unroll
      for (int t = 0; t < NS; ++t) {
        const quad_t a0 = KT::column_quad(kt, at, 32 * kk, t, l15, l4), a1 = KT::column_quad(kt, at, 32 * kk + 16, t, l15, l4);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) S[t] = mma_quads(a0, a1, us[2 * kk][o], us[2 * kk + 1][o], S[t]);
      }
    __syncthreads();
  }
  if (matrix) {
    float* m = seg_at(idx) + DK * p.dv + dv0 + 16 * wave + l15;
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) m[(16 * t + 4 * l4 + r) * DK] = S[t][r];
  } else if (!OUTPUT) {
    keep(idx);
  } else if (idx == nseg - 1) {
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) own[sbase + (uint32_t)((16 * t + r) * p.dv)] = S[t][r];
  }
}

// ---- from a portion's segments (M_i, C_i) to the states behind them, S_i = M_i S_(i-1) + C_i, in place of C_i.  One workgroup per
// 16 columns; a wave owns a quarter of the rows, the operands of S pass through LDS ----
template <int DK>
__global__ __launch_bounds__(256) void delta_chain_kernel(DeltaArgs p) {
  constexpr int NS = DK / 16, TB = NS / 4;
  __shared__ __attribute__((aligned(16))) quad_t sq[NOPND][NS][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int sg = blockIdx.z, h = blockIdx.y, nseg = p.seg[8 * sg + 5];      // (those with work are neighbours: on all XCDs)
  if (p.seg[8 * sg + 4] != 0 || nseg < 3) return;
  const int64_t stride = (int64_t)DK * (p.dv + DK);
  float* at = p.seg_state + ((int64_t)sg * p.H + h) * stride;
  const int64_t next = stride * p.H;                     // to the next segment's
  const uint32_t c0 = 16 * blockIdx.x * DK + 64 * 4 * TB * wave + 4 * lane;
  f32x4 N[TB];
  auto share = [&] {
#pragma unroll
    for (int t = 0; t < TB; ++t) {
      quad_t q[NOPND];
      split_quad(N[t], q);
#pragma unroll
      for (int o = 0; o < NOPND; ++o) sq[o][TB * wave + t][lane] = q[o];
    }
  };
#pragma unroll
  for (int t = 0; t < TB; ++t) N[t] = *(const f32x4*)(at + (c0 + 256 * t));
  share();
  for (int i = 1; i < nseg - 1; ++i) {
    at += next;
    const float* m = at + DK * p.dv;
#pragma unroll
    for (int t = 0; t < TB; ++t) N[t] = *(const f32x4*)(at + (c0 + 256 * t));
    f32x4 a[TB][NS];
#pragma unroll
    for (int t = 0; t < TB; ++t)
#pragma unroll
      for (int k = 0; k < NS; ++k) a[t][k] = *(const f32x4*)(m + (uint32_t)((16 * (TB * wave + t) + l15) * DK + 16 * k + 4 * l4));
    __syncthreads();
#pragma unroll
    for (int k = 0; k < NS; k += 2)
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        quad_t a0[NOPND], a1[NOPND];
        split_quad(a[t][k], a0);
        split_quad(a[t][k + 1], a1);
#pragma unroll
        for (int o = 0; o < NOPND; ++o) N[t] = mma_quads(a0[0], a1[0], sq[o][k][lane], sq[o][k + 1][lane], N[t]);
        if constexpr (SPLIT) N[t] = mma_quads(a0[NOPND - 1], a1[NOPND - 1], sq[0][k][lane], sq[0][k + 1][lane], N[t]);
      }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < TB; ++t) *(f32x4*)(at + (c0 + 256 * t)) = N[t];
    share();
  }
}

// ---- one token per sequence ----
struct DeltaDecodeArgs {
  const elem_t* x; int64_t ld;
  elem_t* o; int64_t ldo;
  float* state;
  float* ring;
  const int *slot, *pos;                 // pos < 0: an empty place of the batch
  const float* conv_w; int taps;
  float qk_eps, scale;
  int64_t ab_col;
  const float *a_log, *dt_bias;
  int64_t g_col;
  const float* w;
  int n;
  float eps;
  int H, G;
};

template <int DK, int DV>
__global__ __launch_bounds__(4 * DV) void delta_decode_kernel(DeltaDecodeArgs p) {
  constexpr int TH = 4 * DV, COLS = DV / 4, ROWS = DK / STATE_GROUPS;
  __shared__ __attribute__((aligned(16))) float qkv[2 * DK + DV];
  __shared__ float unit[2];
  __shared__ f32x4 red[2][STATE_GROUPS][COLS];
  const int b = blockIdx.x, h = blockIdx.y, g = h / (p.H / p.G), tid = threadIdx.x, col = tid % COLS, grp = tid / COLS;
  const int ps = p.pos[b];
  if (ps < 0) return;
  const int slot = p.slot[b], channels = 2 * p.G * DK + p.H * DV;
  const elem_t* row = p.x + (int64_t)b * p.ld;
  float* S = p.state + ((int64_t)slot * p.H + h) * DK * DV + 4 * col + (int64_t)grp * ROWS * DV;
  f32x4 s[ROWS];                         // requested before anything waits
#pragma unroll
  for (int i = 0; i < ROWS; ++i) s[i] = ps > 0 ? *(const f32x4*)(S + (int64_t)i * DV) : zero4();
  // convolution of this head's channels.  The ring has a row more than the inputs it is asked for: the new input (stored by every
  // head that uses it, equal bytes) replaces none that another workgroup still reads.
  float* ring = p.ring + (int64_t)slot * p.taps * channels;
  for (int i = tid; i < 2 * DK + DV; i += TH) {
    const int c = i < DK ? g * DK + i : i < 2 * DK ? (p.G + g) * DK + i - DK : 2 * p.G * DK + h * DV + i - 2 * DK;
    const float in = (float)row[c];
    float y = p.conv_w[(int64_t)(p.taps - 1) * channels + c] * in;
    for (int j = 1; j < min(p.taps, ps + 1); ++j)
      y += p.conv_w[(int64_t)(p.taps - 1 - j) * channels + c] * ring[(int64_t)((ps - j) % p.taps) * channels + c];
    qkv[i] = (float)(elem_t)silu(y);
    if (p.taps > 1) ring[(int64_t)(ps % p.taps) * channels + c] = in;
  }
  const elem_t* ab = row + p.ab_col;
  const float decay = __builtin_amdgcn_exp2f(-__expf(p.a_log[h]) * softplus((float)ab[h] + p.dt_bias[h]) * LOG2E);
  const float beta = sigmoid((float)ab[p.H + h]);
  __syncthreads();
  if (tid < 128) {                       // wave 0: q, wave 1: k
    const float* v = qkv + (tid >> 6) * DK;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < DK; i += 64) ss += v[i + (tid & 63)] * v[i + (tid & 63)];
    ss = wave_sum(ss);
    if ((tid & 63) == 0) unit[tid >> 6] = (tid < 64 ? p.scale : 1.0f) / sqrtf(ss + p.qk_eps);
  }
  __syncthreads();
  const float rq = unit[0], rk = unit[1];
  f32x4 acc = zero4();
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    s[i] *= decay;
    acc += qkv[DK + grp * ROWS + i] * s[i];
  }
  const f32x4 u = beta * (*(const f32x4*)(qkv + 2 * DK + 4 * col) - rk * over_groups<DV>(acc, red[0], grp, col));
  acc = zero4();
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    s[i] += (rk * qkv[DK + grp * ROWS + i]) * u;
    acc += qkv[grp * ROWS + i] * s[i];
    *(f32x4*)(S + (int64_t)i * DV) = s[i];
  }
  const f32x4 y = rq * over_groups<DV>(acc, red[1], grp, col);
  if (tid < COLS) {
    const HeadOut out{row + p.g_col + (int64_t)h * DV, p.w, p.n, p.eps};
    head_out<DV>(y, out, p.o + (int64_t)b * p.ldo + (int64_t)h * DV);
  }
}

template <int DK>
static int launch(const DeltaArgs& a, int segments, int multi, int n_chunks, hipStream_t s) {
  const int channels = 2 * a.G * DK + a.H * a.dv;
  const dim3 cgrid(n_chunks * (DC / CONV_TOKENS), (channels + 256 * FR - 1) / (256 * FR));
  switch (a.taps) {
    case 1: hipLaunchKernelGGL(delta_conv_kernel<1>, cgrid, dim3(256), 0, s, a); break;
    case 2: hipLaunchKernelGGL(delta_conv_kernel<2>, cgrid, dim3(256), 0, s, a); break;
    case 3: hipLaunchKernelGGL(delta_conv_kernel<3>, cgrid, dim3(256), 0, s, a); break;
    case 4: hipLaunchKernelGGL(delta_conv_kernel<4>, cgrid, dim3(256), 0, s, a); break;
    default: hipLaunchKernelGGL(delta_conv_kernel<0>, cgrid, dim3(256), 0, s, a);
  }
  hipLaunchKernelGGL((delta_chunk_kernel<DK>), dim3(a.H, n_chunks), dim3(64), 0, s, a);
  if (multi) {
    auto k = delta_prefill_kernel<DK, false>;
    constexpr size_t lds = DeltaGeom<DK, false>::LDS;
    if (allow_lds(k, lds)) return LM_EINVAL;
    hipLaunchKernelGGL(k, dim3(segments, a.H, (a.dv + DK) / 64), dim3(256), lds, s, a);
    hipLaunchKernelGGL(delta_chain_kernel<DK>, dim3(a.dv / 16, a.H, segments), dim3(256), 0, s, a);
  }
  auto k = delta_prefill_kernel<DK, true>;
  constexpr size_t lds = DeltaGeom<DK, true>::LDS;
  if (allow_lds(k, lds)) return LM_EINVAL;
  hipLaunchKernelGGL(k, dim3(segments, a.H, a.dv / 64), dim3(256), lds, s, a);
  return launch_status();
}

}  // namespace lm

using namespace lm;

extern "C" int lm_delta_chunk_rows(void) { return DC; }
extern "C" int64_t lm_delta_mat_elems(void) { return MATS; }

extern "C" int lm_delta_prefill(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* ring, float* seg_state,
                                const int* portion, const int* chunks, int n_chunks, const int* seg, int segments, int multi,
                                const float* conv_w, int taps, float qk_eps, float scale,
                                int64_t ab_col, const float* a_log, const float* dt_bias, void* y, float* norms, void* mats, float* vecs,
                                int H, int G, int dk, int dv, void* stream) {
  if (segments <= 0 || n_chunks > 65535 || n_chunks < segments || (multi && !seg_state) || H <= 0 || G <= 0 || H % G || dv <= 0 || dv % 64 || taps <= 0 || ldo > (1 << 24) || ld % FR || ldo % 4 || !y ||
      !norms || !mats || !vecs)
    return LM_EINVAL;
  DeltaArgs a{(const elem_t*)x, ld, (elem_t*)o, ldo, state, ring, portion, chunks, seg, seg_state, conv_w, taps, qk_eps, scale, ab_col, a_log, dt_bias,
              (elem_t*)y, norms, (elem_t*)mats, vecs, H, G, dk, dv};
  hipStream_t s = (hipStream_t)stream;
  if (dk == 64) return launch<64>(a, segments, multi, n_chunks, s);
  if (dk == 128) return launch<128>(a, segments, multi, n_chunks, s);
  if (dk == 256) return launch<256>(a, segments, multi, n_chunks, s);
  return LM_EINVAL;
}

extern "C" int lm_delta_decode(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* ring, const int* slot,
                               const int* pos, const float* conv_w, int taps, float qk_eps, float scale, int64_t ab_col,
                               const float* a_log, const float* dt_bias, int64_t g_col, const float* w, int n, float eps, int B, int H,
                               int G, int dk, int dv, void* stream) {
  if (B <= 0 || H <= 0 || G <= 0 || H % G || taps <= 0 || n <= 0 || n > dv || ld % 4 || ldo % 4 || g_col % 4) return LM_EINVAL;
  DeltaDecodeArgs a{(const elem_t*)x, ld, (elem_t*)o, ldo, state, ring, slot, pos, conv_w, taps, qk_eps, scale, ab_col, a_log, dt_bias,
                    g_col, w, n, eps, H, G};
  hipStream_t s = (hipStream_t)stream;
#define LM_CASE(K, V)                                                                                        \
  if (dk == K && dv == V) {                                                                                  \
    hipLaunchKernelGGL((delta_decode_kernel<K, V>), dim3(B, H), dim3(4 * V), 0, s, a);                       \
    return launch_status();                                                                                  \
  }
  LM_CASE(64, 64) LM_CASE(64, 128) LM_CASE(64, 256) LM_CASE(128, 64) LM_CASE(128, 128) LM_CASE(128, 256)
  LM_CASE(256, 64) LM_CASE(256, 128) LM_CASE(256, 256)
#undef LM_CASE
  return LM_EINVAL;
}
