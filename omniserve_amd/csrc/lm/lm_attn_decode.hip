// Decode attention over the paged cache: one new token per sequence.  A workgroup serves up to 16 query heads of one kv head
// (they are the columns of the MFMA tiles) and one part of the visible keys; its four waves take 32-key tiles in turn and
// meet in LDS.  The step in front of it is part of the launch: q and k are turned by their position, the values mixed with the
// first mixing layer's, and the new k / v row appended to its page by the workgroup that owns the newest key.  With one part
// the output leaves gated and normalised; with several, lm_attn_merge_kernel finishes.
#include "lm_attn.h"
#include "omniserve_lm.h"

namespace lm {

struct DecodeArgs {
  const elem_t* qkv; int64_t ld;               // row: q [H][dk], k [G][dk], v [G][dv] as projected
  const elem_t* v_first; int64_t ldv; float lambda;
  const float* freq; int half;
  const int* pos; const int* slot;             // of each sequence's new token; pos < 0: an empty place of the batch
  elem_t* kc; elem_t* vc;
  const int* bt; int bt_stride;                // block table row i belongs to sequence i
  const elem_t* gate; int64_t ldg;
  elem_t* o; int64_t ldo;
  float* part;                                 // nsplit > 1: [B][H][nsplit][dv + 2]
  float scale;
  int window, H, G, nsplit;
};

__device__ __forceinline__ frag_t turn(frag_t v, int d, int pos, const float* freq, int half) {
#pragma unroll
  for (int e = 0; e < FR; e += 2) {
    const int pr = (d + e) >> 1;
    if (pr < half) {
      float s, c;
      sincosf((float)pos * freq[pr], &s, &c);
      const float a = (float)v[e], b = (float)v[e + 1];
      v[e] = (elem_t)(a * c - b * s);
      v[e + 1] = (elem_t)(b * c + a * s);
    }
  }
  return v;
}

template <int DK, int DV>
__global__ __launch_bounds__(256) void attn_decode_kernel(DecodeArgs p) {
#if LM_ELEM == 0
  typedef Tile<DV * (int)sizeof(elem_t)> VT;
#endif
  constexpr int NKF = DK / KSTEP, NVB = DV / 16, VTILE = 32 * DV * (int)sizeof(elem_t);
  constexpr int RED = 4 * 16 * (DV + 4) * 4;
  __shared__ __attribute__((aligned(16))) uint8_t lds[SPLIT && 4 * VTILE > RED ? 4 * VTILE : RED];   // V tiles (bf16), then the waves' results
  __shared__ __attribute__((aligned(16))) elem_t qs[16][DK];
  __shared__ float wm[4][16], wl[4][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l15 = lane & 15, l4 = lane >> 4;
  const int b = blockIdx.x, gs = p.H / p.G, hb = (gs + 15) / 16, g = blockIdx.y / hb, h0 = g * gs + 16 * (blockIdx.y % hb);
  const int nh = min(16, (g + 1) * gs - h0), split = blockIdx.z;
  const int pos = p.pos[b];
  if (pos < 0) return;
  const int lo = max(0, pos - p.window + 1), t0 = lo >> 5, nt = (pos >> 5) - t0 + 1, per = (nt + p.nsplit - 1) / p.nsplit;
  const int ta = t0 + split * per, tb = min(t0 + nt, ta + per);
  const int* bt = p.bt + (int64_t)b * p.bt_stride;
  const elem_t* row = p.qkv + (int64_t)b * p.ld;

  for (int i = tid; i < nh * (DK / FR); i += 256) {
    const int hh = i / (DK / FR), d = (i - hh * (DK / FR)) * FR;
    *(frag_t*)&qs[hh][d] = turn(*(const frag_t*)(row + (int64_t)(h0 + hh) * DK + d), d, pos, p.freq, p.half);
  }
  for (int i = tid; i < (16 - nh) * (DK / FR); i += 256) *(frag_t*)&qs[nh + i / (DK / FR)][i % (DK / FR) * FR] = frag_t{};
  // the new key and value: written by every workgroup of this kv head that reads them itself (equal bytes), i.e. by the one
  // part that holds the newest tile
  const int slot = p.slot[b];
  if (tb == t0 + nt && ta < tb && slot >= 0) {
    const int64_t page = slot / PAGE;
    const int at = slot % PAGE;
    for (int i = tid; i < DK / FR; i += 256) {
      const int d = i * FR;
      *(frag_t*)(p.kc + ((page * p.G + g) * PAGE + at) * DK + d) =
          turn(*(const frag_t*)(row + (int64_t)(p.H + g) * DK + d), d, pos, p.freq, p.half);
    }
    for (int i = tid - 128; i >= 0 && i < DV / FR; i += 128) {
      const int d = i * FR;
      frag_t v = *(const frag_t*)(row + (int64_t)(p.H + p.G) * DK + (int64_t)g * DV + d);
      if (p.v_first) {
        const frag_t f = *(const frag_t*)(p.v_first + (int64_t)b * p.ldv + (int64_t)g * DV + d);
#pragma unroll
        for (int e = 0; e < FR; ++e) v[e] = (elem_t)((1.0f - p.lambda) * (float)v[e] + p.lambda * (float)f[e]);
      }
      *(frag_t*)(p.vc + ((page * p.G + g) * PAGE + at) * DV + d) = v;
    }
  }
  __syncthreads();      // (also makes the appended row visible to the other waves of this workgroup)

  frag_t qf[NKF];
#pragma unroll
  for (int s = 0; s < NKF; ++s) qf[s] = *(const frag_t*)&qs[l15][s * KSTEP + FR * l4];
  f32x4 acc[NVB];
#pragma unroll
  for (int c = 0; c < NVB; ++c) acc[c] = zero4();
  float m_run = NEG, l_run = 0.f;
#if LM_ELEM == 0
  uint8_t* vt = lds + wave * VTILE;
#endif
  for (int t = ta + wave; t < tb; t += 4) {
    const int kb = 32 * t;
    const int64_t page = bt[kb / PAGE];
    const elem_t* kp = p.kc + ((page * p.G + g) * PAGE + kb % PAGE) * DK;
    const elem_t* vp = p.vc + ((page * p.G + g) * PAGE + kb % PAGE) * DV;
    frag_t kf[2][NKF];
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int s = 0; s < NKF; ++s) kf[u][s] = *(const frag_t*)(kp + (16 * u + l15) * DK + s * KSTEP + FR * l4);
#if LM_ELEM == 0
    frag_t vf[VTILE / 1024];
#pragma unroll
    for (int i = 0; i < VTILE / 1024; ++i) vf[i] = *(const frag_t*)(vp + (64 * i + lane) * FR);
#endif
    f32x4 x[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      x[u] = zero4();
#pragma unroll
      for (int s = 0; s < NKF; ++s) x[u] = mma(kf[u][s], qf[s], x[u]);
    }
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = kb + 16 * u + 4 * l4 + r;
        x[u][r] = (int)(key <= pos) & (int)(key >= lo) ? x[u][r] : NEG;
      }
    quad_t pq[2][NOPND];
    const float alpha = softmax_step<2>(x, p.scale, m_run, l_run, pq);
#pragma unroll
    for (int c = 0; c < NVB; ++c) acc[c] *= alpha;
#if LM_ELEM == 0
    __builtin_amdgcn_wave_barrier();       // LDS operations of one wave are in order: the previous tile has been read
#pragma unroll
    for (int i = 0; i < VTILE / 1024; ++i) {
      const int sl = 64 * i + lane;
      *(frag_t*)(vt + VT::slot(sl / VT::NS, sl % VT::NS)) = vf[i];
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#endif
#pragma unroll
    for (int c = 0; c < NVB; ++c) {
      quad_t v0, v1;
#if LM_ELEM == 0
      v0 = VT::column_quad(vt, 0, c, l15, l4);
      v1 = VT::column_quad(vt, 16, c, l15, l4);
#else
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        v0[i] = vp[(4 * l4 + i) * DV + 16 * c + l15];
        v1[i] = vp[(16 + 4 * l4 + i) * DV + 16 * c + l15];
      }
#endif
#pragma unroll
      for (int o = 0; o < NOPND; ++o) acc[c] = mma_quads(v0, v1, pq[0][o], pq[1][o], acc[c]);
    }
  }
  l_run = column_sum(l_run);
  __syncthreads();      // every wave is done with its V tile
  float(*res)[16][DV + 4] = (float(*)[16][DV + 4])lds;
#pragma unroll
  for (int c = 0; c < NVB; ++c) *(f32x4*)&res[wave][l15][16 * c + 4 * l4] = acc[c];
  if (l4 == 0) { wm[wave][l15] = m_run; wl[wave][l15] = l_run; }
  __syncthreads();
  for (int i = tid; i < nh * (DV / 4); i += 256) {
    const int hh = i / (DV / 4), d = (i - hh * (DV / 4)) * 4;
    const float m = fmaxf(fmaxf(wm[0][hh], wm[1][hh]), fmaxf(wm[2][hh], wm[3][hh]));
    f32x4 y = zero4();
    float l = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = __builtin_amdgcn_exp2f(wm[w][hh] - m);
      l += f * wl[w][hh];
      y += f * *(const f32x4*)&res[w][hh][d];
    }
    if (p.nsplit > 1) {
      float* q = p.part + (((int64_t)b * p.H + h0 + hh) * p.nsplit + split) * (DV + 2);
#pragma unroll
      for (int r = 0; r < 4; ++r) q[2 + d + r] = y[r];
      if (d == 0) { q[0] = m; q[1] = l; }
    } else {
      y *= 1.0f / l;
      if (p.gate) {
        const f32x4 z = from_quad(*(const quad_t*)(p.gate + (int64_t)b * p.ldg + (int64_t)(h0 + hh) * DV + d));
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] *= sigmoid(z[r]);
      }
      *(quad_t*)(p.o + (int64_t)b * p.ldo + (int64_t)(h0 + hh) * DV + d) = to_quad(y);
    }
  }
}

template <int DK, int DV>
static int launch(const DecodeArgs& a, int B, hipStream_t s) {
  const int gs = a.H / a.G, hb = (gs + 15) / 16;
  hipLaunchKernelGGL((attn_decode_kernel<DK, DV>), dim3(B, a.G * hb, a.nsplit), dim3(256), 0, s, a);
  if (a.nsplit > 1)
    hipLaunchKernelGGL(attn_merge_kernel, dim3(B, a.H), dim3(256), 0, s, a.part, a.nsplit, a.pos, a.gate, a.ldg, a.o, a.ldo, a.H, DV);
  return launch_status();
}

}  // namespace lm

using namespace lm;

extern "C" int lm_attn_decode(const void* qkv, int64_t ld, const void* v_first, int64_t ldv, float lambda, const float* freq, int half,
                              const int* pos, const int* slot, void* kc, void* vc, const int* bt, int bt_stride, const void* gate,
                              int64_t ldg, void* o, int64_t ldo, float* part, int nsplit, float scale, int window, int B, int H, int G,
                              int dk, int dv, void* stream) {
  if (B <= 0 || G <= 0 || H % G || !(scale > 0.f) || window <= 0 || half < 0 || 2 * half > dk || nsplit <= 0 || (nsplit > 1 && !part) ||
      ld % FR || ldv % FR || ldo % 4 || ldg % 4 || nsplit > 64)
    return LM_EINVAL;
  DecodeArgs a{(const elem_t*)qkv, ld, (const elem_t*)v_first, ldv, lambda, freq, half, pos, slot, (elem_t*)kc, (elem_t*)vc, bt, bt_stride,
               (const elem_t*)gate, ldg, (elem_t*)o, ldo, part, scale * 1.4426950408889634f, window, H, G, nsplit};
  hipStream_t s = (hipStream_t)stream;
#define LM_CASE(K, V) if (dk == K && dv == V) return launch<K, V>(a, B, s);
  LM_CASE(64, 64) LM_CASE(64, 128) LM_CASE(64, 256) LM_CASE(128, 64) LM_CASE(128, 128) LM_CASE(128, 256)
  LM_CASE(256, 64) LM_CASE(256, 128) LM_CASE(256, 256)
#undef LM_CASE
  return LM_EINVAL;
}
