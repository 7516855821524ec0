/* C ABI of the serving engine's layer kernels (libomniserve_lm_bf16.so, libomniserve_lm_f32.so: the same entry points for one
 * element type each).  Device pointers, sizes, strides in elements, a hipStream_t; every call only enqueues (no allocation, no
 * synchronisation).  Returns 0, -22 (arguments) or -5 (launch).  "elem" is the library's element type.
 *
 * Conventions of the callers' data: inner sizes are padded with zeros to multiples of 64 (model width, feed-forward, and per
 * head to 64 / 128 / 256), so that no kernel guards a k loop; statistics take the real size as an argument. */
#pragma once
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define LM_ABI_VERSION 3
#define LM_NORM_LAYER 0
#define LM_NORM_RMS 1
#define LM_EPI_ELEM 0
#define LM_EPI_F32 1
#define LM_EPI_GLU 2
#define LM_EPI_GATE 3
#define LM_ACT_NONE 0
#define LM_ACT_SILU 1
#define LM_ACT_GELU_TANH 2
#define LM_ACT_SIGMOID 3
#define LM_TILE_ROWS 256 /* rows of one lm_gemm_tiles tile */
#define LM_ATTN_ROWS 128 /* query rows of one lm_attn_prefill tile */

int lm_abi_version(void);
int lm_elem_bytes(void);

/* Residual stream x (f32) and the norms around it, one token per row:
 *   x = embed_scale * embed[tokens]        (tokens given)
 *   y = sublayer output (+ y_bias), or the weighted sum of its expert rows (top > 0)
 *   x += norm(y; post_w, post_b)           (post_w null: x += y;  y null: nothing added)
 *   h = norm(x; next_w, next_b)            (next_w null: h = x;  h null: none)
 * kind: LM_NORM_LAYER / LM_NORM_RMS over the first n columns.  Expert rows: (token, choice) pair t * top + k of y, weight
 * pair_w of the same index; shared != 0: row pairs0 + t is added with weight one.  rows: row r of h belongs to token rows[r]. */
int lm_residual_norm(float* x, int64_t ldx, const int* tokens, const void* embed, float embed_scale, const void* y, int64_t ldy,
                     const float* y_bias, const float* pair_w, int top, int pairs0, int shared, const float* post_w, const float* post_b, const float* next_w,
                     const float* next_b, void* h, int64_t ldh, const int* rows, int n_rows, int n, int kind, int store_x, float eps,
                     void* stream);

/* out = rms_norm(o) * w * sigmoid(gate); n real columns of cols */
int lm_gated_rms(void* out, int64_t ldo, const void* o, int64_t ldi, const void* gate, int64_t ldg, const float* w, int rows, int cols,
                 int n, float eps, void* stream);

/* Rows q [H][dk] k [G][dk] v [G][dv]: q, k turned in place / into the cache, v mixed ((1 - lambda) v + lambda v_first) into the
 * cache.  freq: rotation per position of each of the `half` pairs.  slot = page * 64 + offset, < 0: not stored. */
int lm_rope_append(void* qkv, int64_t ld, const void* v_first, int64_t ldv, float lambda, const float* freq, int half, const int* pos,
                   const int* slot, void* kc, void* vc, int tokens, int H, int G, int dk, int dv, void* stream);

/* Causal sliding-window attention of prompt portions over pages of 64 keys and values: the row of key i of kv head g in page p
 * starts at kc + p * k_page + g * k_head + i * k_row (values alike).  The cache's pools [page][G][64][dk | dv] are one such layout,
 * rows [tokens][G][dk | dv] another.  entry [.][4]: first token, tokens, position of the first token, block table row; tiles
 * [n_tiles][2]: entry, first row. */
int lm_attn_prefill(const void* q, int64_t ldq, const void* kc, int64_t k_page, int k_head, int k_row, const void* vc,
                    int64_t v_page, int v_head, int v_row, const int* bt, int bt_stride, const int* entry,
                    const int* tiles, int n_tiles, const void* gate, int64_t ldg, void* o, int64_t ldo, float scale, int window, int H,
                    int G, int dk, int dv, void* stream);

/* One token per sequence: rotation + value mixing + append + attention + gate.  part: f32 [B][H][nsplit][dv + 2] for nsplit > 1. */
int lm_attn_decode(const void* qkv, int64_t ld, const void* v_first, int64_t ldv, float lambda, const float* freq, int half,
                   const int* pos, const int* slot, void* kc, void* vc, const int* bt, int bt_stride, const void* gate, int64_t ldg,
                   void* o, int64_t ldo, float* part, int nsplit, float scale, int window, int B, int H, int G, int dk, int dv,
                   void* stream);

/* Decayed linear attention; rows q [H][dk] k [H][dk] v [H][dv], `act` applied to all three.  seg [.][8]: first token, tokens,
 * slot, starts from zero, index in its entry, segments of the entry, 0, 0; all but an entry's last have seg_len tokens.
 * multi: some entry has several segments (seg_state: f32 [segments][H][dk][dv]). */
int lm_linear_prefill(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* seg_state, const int* seg, int segments,
                      int seg_len, int multi, const float* log2_decay, int H, int dk, int dv, int act, void* stream);
int lm_linear_decode(const void* x, int64_t ld, void* o, int64_t ldo, float* state, const int* slot, const int* pos,
                     const float* log2_decay, int B, int H, int dk, int dv, int act, void* stream);

/* ---- latent attention: a cache row per token [Rp | Tp] = (normed latent, turned key part), one pool [pages][64][Rp + Tp] ----
 * Rotation here pairs dimension i with i + half.  Query rows: H heads of dk, the turned part (2 * half) from column q_rot on. */
/* x: q [H][dk] ..., at column src_col the projection of the cache row ([Rp | Tp], R real latent columns).  Turns q in place; with
 * src_col >= 0 also norms (weight w, eps) and turns the row and stores it at slot. */
int lm_latent_append(void* x, int64_t ld, int64_t src_col, const float* w, float eps, const float* freq, int half, const int* pos,
                     const int* slot, void* cache, int tokens, int H, int dk, int q_rot, int R, int Rp, int Tp, void* stream);
/* dst[i] = src[pages[i]], pages of 64 * row elements */
int lm_gather_pages(void* dst, const void* src, const int* pages, int n_pages, int row, void* stream);
/* One token per sequence: append (src_col >= 0) + turn q + attention over the cache rows; qa: the queries' unturned parts taken into
 * the latent space [B][H][Rp]; o [B][H][Rp]: weighted sums of latents.  part: f32 [B][H][nsplit][Rp + 2] for nsplit > 1. */
int lm_latent_decode(const void* x, int64_t ld, int64_t src_col, const float* w, float eps, const float* freq, int half, const int* pos,
                     const int* slot, void* cache, const int* bt, int bt_stride, const void* qa, void* o, float* part, int nsplit,
                     float scale, int B, int H, int dk, int q_rot, int R, int Rp, int Tp, void* stream);

/* out = act(gate + bias) * (up + bias) of rows x in alternating blocks of 16 gate / 16 up channels (n of both) */
int lm_glu(void* out, int64_t ldo, const void* x, int64_t ldx, const float* bias, int rows, int n, int act, void* stream);

/* out = rms_norm(o per head over n of its dv columns) * w [dv] * act(gate); act: LM_ACT_SILU / LM_ACT_SIGMOID */
int lm_gated_head_rms(void* out, int64_t ldo, const void* o, int64_t ldi, const void* gate, int64_t ldg, const float* w, int rows, int H,
                      int dv, int n, float eps, int act, void* stream);

/* ---- gated linear attention: S <- diag(alpha) S + k v^T, o = scale S^T q, alpha = sigmoid(low a2^T + bias)^(1 / tau) per key
 * channel.  Rows: q [H][dk] k [H][dk] v [H][dv]; the decays' low-rank input (rp columns) at column low_col; a2 [H * dk][rp]; bias
 * [H * dk].  seg, seg_len, multi, seg_state as in lm_linear_prefill; seg_decay: f32 [segments][H][dk]. */
int lm_gla_prefill(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* seg_state, float* seg_decay, const int* seg,
                   int segments, int multi, int64_t low_col, const void* a2, const float* bias, int rp, float inv_tau, float scale, int H,
                   int dk, int dv, void* stream);
/* + RMS norm per head over n columns (w, eps) and silu(gate at column g_col) */
int lm_gla_decode(const void* x, int64_t ld, void* o, int64_t ldo, float* state, const int* slot, const int* pos, int64_t low_col,
                  const void* a2, const float* bias, int rp, float inv_tau, float scale, int64_t g_col, const float* w, int n, float eps,
                  int B, int H, int dk, int dv, void* stream);

/* ---- gated delta rule: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  Rows: q [G][dk] k [G][dk] v [H][dv] as projected;
 * a, b (H each) at column ab_col.  Every channel of q, k, v passes a causal convolution of `taps` inputs (conv_w [taps][channels],
 * last row: the current input) and silu; q and k become unit vectors (eps qk_eps), q times scale.  ring: f32 [slots][taps][channels],
 * the input of position p in row p % taps.
 * portion [.][8]: first token, tokens, slot, starts from zero, first chunk, chunks, position, 0; chunks [n_chunks]: portion of every
 * chunk of lm_delta_chunk_rows() tokens.  seg, multi as in lm_linear_prefill, every segment of whole chunks but a portion's last, its
 * first chunk in column 6; seg_state: f32 [segments][H][dk * (dv + dk)].  y: the convolved rows [tokens][channels], norms: f32 [tokens][2 G], mats: elem
 * [n_chunks][H][2][operands][rows][rows], vecs: f32 [n_chunks][H][4][rows]. */
int lm_delta_chunk_rows(void);
int64_t lm_delta_mat_elems(void);
int lm_delta_prefill(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* ring, float* seg_state, const int* portion,
                     const int* chunks, int n_chunks, const int* seg, int segments, int multi, const float* conv_w, int taps, float qk_eps, float scale, int64_t ab_col,
                     const float* a_log, const float* dt_bias, void* y, float* norms, void* mats, float* vecs, int H, int G, int dk,
                     int dv, void* stream);
int lm_delta_decode(const void* x, int64_t ld, void* o, int64_t ldo, float* state, float* ring, const int* slot, const int* pos,
                    const float* conv_w, int taps, float qk_eps, float scale, int64_t ab_col, const float* a_log, const float* dt_bias,
                    int64_t g_col, const float* w, int n, float eps, int B, int H, int G, int dk, int dv, void* stream);

/* z [tokens][ldz] f32 router logits -> wts [tokens][top], off [experts + 1], perm [tokens * top] (pairs sorted by expert);
 * with tiles: [lm_route_max_tiles][4] (expert, first place, rows, 0) of every row tile, rows = 0 past the last. */
int64_t lm_route_scratch_words(int tokens, int experts, int top);
int lm_route_max_tiles(int tokens, int experts, int top);
int lm_route(const float* z, int64_t ldz, const float* bias, int tokens, int experts, int top, float* wts, int* off, int* perm,
             int* tiles, int* scratch_i32, void* stream);

/* y = x w^T for one or many matrices w [groups][n][k].  perm null: rows_a rows, group g reads x from column g * gx and writes y
 * from column g * gy (several groups: lm_gemm_rows only).  Else group g has the places off[g] .. off[g + 1] of perm; a place's y
 * row is perm[place], its x row perm[place] / x_div.  b (optional): one more matrix over rows 0 .. rows_b - 1 of its own x and y.
 * epi: LM_EPI_ELEM; LM_EPI_F32 (times scale); LM_EPI_GLU (rows of w in alternating blocks of 16 gate / 16 up channels, bias in the
 * same order; y has n / 2 columns: act(gate + bias) * (up + bias), act LM_ACT_SILU or LM_ACT_GELU_TANH); LM_EPI_GATE (times
 * sigmoid(gate), gate addressed like y with row stride ldg; lm_gemm_rows only). */
typedef struct {
  const void* w;
  const void* x;
  int64_t ldx;
  void* y;
  int64_t ldy;
  int n, k;
  int64_t gx, gy;
  const float* bias;
  const void* gate;
  int64_t ldg;
} LmGemmPart;
int lm_gemm_rows(const LmGemmPart* a, const LmGemmPart* b, int groups, const int* perm, const int* off, int rows_a, int rows_b,
                 int x_div, int max_rows, float scale, int epi, int act, void* stream);
int lm_gemm_tiles(const LmGemmPart* a, const LmGemmPart* b, int groups, const int* perm, const int* off, const int* tiles,
                  int max_tiles, int rows_a, int rows_b, int x_div, float scale, int epi, int act, void* stream);

int lm_argmax(int64_t* out, const float* z, int64_t ld, int rows, int n, void* stream);

#ifdef __cplusplus
}
#endif
