// Launch functions of the floating-point layers (linears, norms, latent attention, attention over shared key/value rows,
// gated linear attention, mixture of experts).  ET is bf16_t or float; every function only enqueues work on `st` and returns a status code.
#pragma once
#include "elem.h"

namespace fx {

// ---- linears over many rows (csrc/gemm_float.hip) --------------------------------------------------------------
// C = A W^T with A [m][lda] and W [n][k] of ET, k a multiple of 64.  Columns below n_split leave as ET in y (with `glu`:
// weight rows 2i / 2i+1 are gate and up of unit i, and the gated unit of the pair leaves in column i); the columns from
// n_split on leave as float32 in y32.  bias [n]: added to every row ahead of all that.  row_src: row r of A is read at row row_src[r].  tiles: grouped form, one weight
// matrix per group (w_stride elements apart); rows of a group are contiguous in C, and tiles[i] = {group, first row,
// end row, 0} for the *n_tiles tiles of `tile_rows` rows each.
struct GemmArgs {
    const void* a = nullptr; const void* w = nullptr;
    int lda = 0, ldw = 0, m = 0, n = 0, k = 0;           // ldw 0: rows of W are k long
    int n_split = 0, glu = 0;
    float limit = 0.0f;
    const float* bias = nullptr;
    void* y = nullptr; int ldy = 0;
    float* y32 = nullptr; int ldy32 = 0;
    const int* row_src = nullptr;
    const int4* tiles = nullptr; const int* n_tiles = nullptr; int max_tiles = 0;
    size_t w_stride = 0;
};
template <typename ET> int gemm_float(const GemmArgs& g, hipStream_t st);
// The grouped form; the table is cut for tiles of tile_rows (64 or 128) rows, gemm_group_tile_rows says which suits.
template <typename ET> int gemm_grouped(const GemmArgs& g, int tile_rows, hipStream_t st);
int gemm_group_tile_rows(int rows_per_group);

// ---- linears of one token (csrc/gemv_float.hip) ----------------------------------------------------------------
// The vector is float32.  Prologue 0: x [tokens][ldx] as it is.  Prologue 1: h = norm(x + normb(y)), where the y part is
// left out when y is null and its norm when gb is null; without gb, x0 [tokens][ldx] (or null) is added as well.  Block 0 of
// a token writes the new residual to x_new and h to h_out (either may be null).
// Prologue 2: like 0 for the experts chosen from router outputs: grid row t*top+i runs expert i of token t (weights
// w + expert * w_stride), the choice and its weights are left in pick / pick_w.
struct GemvArgs {
    const void* w = nullptr;
    int n = 0, k = 0, kpad = 0, n_split = 0, glu = 0;
    float limit = 0.0f;
    const float* x = nullptr; int ldx = 0;
    const float* y = nullptr; int ldy = 0;
    const float *gb = nullptr, *g = nullptr;              // weight of the norm after / before a sublayer
    const float* x0 = nullptr;
    const float* bias = nullptr;                          // [n]
    float eps = 0.0f;
    float *x_new = nullptr, *h_out = nullptr; int ldh = 0;
    float* out = nullptr; int ldo = 0;                    // columns below n_split (after glu)
    float* out32 = nullptr; int ldo32 = 0;                // the others
    const float* route = nullptr; int ld_route = 0, experts = 0, top = 0;
    int* pick = nullptr; float* pick_w = nullptr;
    size_t w_stride = 0;
};
template <typename ET> int gemv_float(const GemvArgs& g, int prologue, int tokens, hipStream_t st);
// y[t] = sum_i pick_w[t][i] * W_down[pick[t][i]] h[t*top+i]  (+ sigmoid(gate) * W_shared hs[t], gate = route[t][experts])
struct MoeDownArgs {
    const void* w = nullptr; size_t w_stride = 0; int kpad = 0, k = 0;
    const float* h = nullptr; int ldh = 0;
    const void* ws = nullptr; int ks_pad = 0, ks = 0;
    const float* hs = nullptr; int ldhs = 0;
    const float* route = nullptr; int ld_route = 0, experts = 0, top = 0;
    const int* pick = nullptr; const float* pick_w = nullptr;
    float* y = nullptr; int ldy = 0, n = 0;
};
template <typename ET> int moe_down_small(const MoeDownArgs& a, int tokens, hipStream_t st);

// ---- rows (csrc/rows_float.hip) --------------------------------------------------------------------------------
template <typename ET> int pack_rows(const bf16_t* src, ET* dst, int n, int k, int kpad, int row_step, int row_off, hipStream_t st);
int widen_rows(const bf16_t* src, float* dst, int n, float add, hipStream_t st);
int embed_rows_bf16(const bf16_t* table, float scale, const int* tokens, int n, float* x, int width, int vocab, int* err, hipStream_t st);
int set_state_launch(int* state, int pos, int step, hipStream_t st);
int advance_launch(int* state, int n, hipStream_t st);
// x += gb * rms(y) (skipped when y is null; plain y when gb is null) + x0 (skipped when null), then h = g * rms(x) (skipped
// when h is null).  The new x goes to x_new, or back to x when that is null.  With a mixture, y is
// gathered: y = sum_i pick_w[t][i] * ys[pos_of[t*top+i]] + sigmoid(route[t][experts]) * y (y, the shared expert's rows,
// may then be null).  rows_src: row r works on x[rows_src[r]] and leaves x alone.
struct RowArgs {
    float *x = nullptr, *x_new = nullptr;
    const float* x0 = nullptr;
    const float* y = nullptr; int ldy = 0;
    const float *gb = nullptr, *g = nullptr;
    float eps = 0.0f;
    int width = 0, rows = 0;
    void* h = nullptr; int ldh = 0; int h_f32 = 0;        // h as float32 instead of ET
    const int* rows_src = nullptr;
    const float* ys = nullptr; const int* pos_of = nullptr; const float* pick_w = nullptr; int top = 0;
    const float* route = nullptr; int ld_route = 0, experts = 0;
};
template <typename ET> int norm_rows(const RowArgs& a, hipStream_t st);

// ---- mixture of experts over many rows (csrc/gemv_float.hip) ------------------------------------------------------------
struct MoePlan { int *pick, *pos_of, *row_src, *counts; float* pick_w; int4* tiles; int* n_tiles; };
// counts: 2 * experts ints.  max tiles = rows * top / tile_rows + experts.
int moe_plan(const float* route, int ld_route, int rows, int experts, int top, int tile_rows, const MoePlan& p, hipStream_t st);

// ---- latent attention (csrc/latent_attn.hip) --------------------------------------------------------------------
// Stored row of a token: [latent, padded to kvp][rotated shared key part, padded], `ldc` elements.
struct LatentDims {
    int heads, dim, rot_dim, vdim, kv_rank, kvp, ldc, window;     // window 0: every earlier position
    float scale, eps;
    int capacity;
};
// Rows of the q / dkv projection: rotates the queries' rotated part in q [tokens][ldq] and leaves the tokens' own rows in
// the cache (raw [tokens][ld_raw] float32; null: the layer has no rows of its own).
template <typename ET> int latent_store(const LatentDims& d, ET* q, int ldq, const float* raw, int ld_raw, const float* norm_w, const float* cos_t,
                                        const float* sin_t, ET* cache, const int* state, int tokens, hipStream_t st);
// Attention over the stored rows themselves: the unrotated query is carried into the latent space through W_uk, the
// context back through W_uv.  Any size; for few tokens.  q as latent_store leaves it.  Scratch:
// latent_absorbed_scratch floats per token.
size_t latent_absorbed_scratch(const LatentDims& d);
template <typename ET> int latent_absorbed(const LatentDims& d, const ET* q, int ldq, const ET* w_uk, const ET* w_uv, const ET* cache,
                                           const int* state, int tok0, int tokens, float* scratch, ET* o, int ldo, hipStream_t st);
// Both in the one-token path: q, raw and o float32, q not rotated yet and left alone.
template <typename ET> int latent_decode(const LatentDims& d, const float* q, int ldq, const float* raw, int ld_raw, const float* norm_w,
                                         const float* cos_t, const float* sin_t, const ET* w_uk, const ET* w_uv, ET* cache, const int* state,
                                         int tokens, float* scratch, float* o, int ldo, hipStream_t st);
// Attention of many tokens with keys and values formed once: k [rows][ldk] (heads x dim), vt [heads x vdim][ldv] for the
// stored rows kv0 .. kv0+rows-1.  bfloat16 only.
bool latent_flash_ok(const LatentDims& d);
int latent_flash(const LatentDims& d, const bf16_t* q, int ldq, const bf16_t* k, int ldk, const bf16_t* vt, int ldv, const bf16_t* cache,
                 int kv0, int pos0, int tokens, bf16_t* o, int ldo, hipStream_t st);

// ---- attention whose values are its projected keys (csrc/shared_kv_attn.hip) ------------------------------------------
// A token leaves one row per key/value head, the projected key: it is the value as it stands, and the key once divided by
// its root mean square, whose reciprocal is stored beside it.  The weights of the query and key norms, the score scale and
// the query's temperature 1 + temp_coef * ln(floor((p + 1) / temp_every) + 1) all multiply the query.  sink: one is added to
// the softmax denominator.  Head rows are `dimp` elements long (pad8(dim), zeros behind dim).
__host__ __device__ constexpr int pad8(int v) { return (v + 7) / 8 * 8; }
struct SharedKvDims {
    int heads, kv_heads, dim, dimp, sink, temp_every, capacity;
    float scale, temp_coef, eps;
};
// A sequence's rows: row [kv_heads][capacity][dimp] of ET, inv_rms [kv_heads][capacity].
template <typename ET> struct SharedKvRows { ET* row; float* inv_rms; };
// Rows of a step into the cache: k [tokens][ldk] float32 (kv_heads x dimp).
template <typename ET> int shared_kv_store(const SharedKvDims& d, const float* k, int ldk, SharedKvRows<ET> c, const int* state, int tokens, hipStream_t st);
// Few tokens (any size): splits of the visible rows, joined by a second kernel.  k as above for tokens whose rows are not in
// the cache yet (they are stored on the way), null when shared_kv_store has been there.  q [tokens][ldq] (heads x dimp),
// not normed, and o [tokens][ldo] (heads x dim) are ET, or float32 with f32.  norm_w [dimp]: product of the two norms'
// weights.  Scratch: shared_kv_scratch floats per token.
size_t shared_kv_scratch(const SharedKvDims& d);
template <typename ET> int shared_kv_splits(const SharedKvDims& d, const void* q, int ldq, const float* k, int ldk, const float* norm_w, SharedKvRows<ET> c,
                                            const int* state, int tok0, int tokens, float* scratch, void* o, int ldo, int f32, hipStream_t st);
// Many tokens on the matrix cores, their rows being in the cache.  bfloat16 only.
bool shared_kv_flash_ok(const SharedKvDims& d);
int shared_kv_flash(const SharedKvDims& d, const bf16_t* q, int ldq, const float* norm_w, SharedKvRows<bf16_t> c, int pos0, int tokens, bf16_t* o, int ldo,
                    hipStream_t st);

// ---- gated linear attention (csrc/gla.hip) -----------------------------------------------------------------------
struct GlaDims { int heads, dim, vdim, a_rank; float tau, eps; };
// p: projections [tokens][ldp] = [q | k | v | g], PT = ET, or float in the one-token path; a1 [tokens][ld_a1] float32;
// state [heads][dim][vdim].  One token after the other, any size.
template <typename ET> int gla_steps(const GlaDims& d, const void* p, int ldp, int p_f32, const float* a1, int ld_a1, const ET* w_a2,
                                     const float* b_a2, const float* norm_w, float* state, const int* pos_state, int tok0, int tokens,
                                     void* o, int ldo, int o_f32, hipStream_t st);
// The same in chunks on the matrix cores (float32).  Scratch floats: gla_chunk_scratch.
bool gla_chunks_ok(const GlaDims& d);
size_t gla_chunk_scratch(const GlaDims& d, int tokens);
template <typename ET> int gla_chunks(const GlaDims& d, const ET* p, int ldp, const float* a1, int ld_a1, const ET* w_a2,
                                      const float* b_a2, const float* norm_w, float* state, const int* pos_state, int tokens,
                                      float* scratch, ET* o, int ldo, hipStream_t st);

}  // namespace fx
