// Attention whose values are its projected keys.  A token leaves one row per key/value head: the projected key, which is the
// value as it stands, and the reciprocal of its root mean square, which turns a product with the row into a product with
// the normed key (the weights of the key norm multiply the query instead).  A row is so read once for score and value.
//
// Few tokens: a workgroup takes a split of the visible rows for up to GH query heads of a key/value head.  16-byte pieces of a
// row live in the registers of LPK neighbouring lanes, which sum the score among themselves and then add the same registers,
// weighted, to their columns; groups of lanes walk over the rows with running maxima of their own and meet at the end.
// Many tokens: flash-style on v_mfma_f32_32x32x16_bf16 with one LDS tile of rows for both products, the second one reading
// it transposed (ds_read_b64_tr_b16).  Scores and weights are float32 throughout: the weights enter the second product as
// the sum of two bfloat16 halves, which keeps 16 bits of each.
//
// Scores are kept in units of log 2, so that weights are powers of two.
#include "float_ops.h"

namespace fx {

constexpr float kLog2e = 1.44269504088896340736f;

// What multiplies the normed query of position pos besides the norms' weights.
__device__ __forceinline__ float query_factor(const SharedKvDims& d, int pos) {
    float f = d.scale * kLog2e;
    if (d.temp_coef != 0.0f) f *= 1.0f + d.temp_coef * logf((float)((pos + 1) / d.temp_every) + 1.0f);
    return f;
}

// Sum over groups of N neighbouring lanes; every lane gets its group's.
template <int N>
__device__ __forceinline__ float group_sum(float v) {
    if constexpr (N > 1) v += lane_xor_f<1>(v);
    if constexpr (N > 2) v += lane_xor_f<2>(v);
    if constexpr (N > 4) v += lane_xor_f<4>(v);
    if constexpr (N > 8) v += lane_xor_f<8>(v);
    if constexpr (N > 16) v += lane_xor_f<16>(v);
    if constexpr (N > 32) v += lane_xor_f<32>(v);
    return v;
}

// ---- rows of a step into the cache: LPR lanes per row -------------------------------------------------------------
template <typename ET, int LPR>
__global__ __launch_bounds__(256) void shared_kv_store_kernel(SharedKvDims d, const float* __restrict__ k, int ldk, SharedKvRows<ET> c,
                                                              const int* __restrict__ state, int total) {
    const int n = blockIdx.x * (256 / LPR) + threadIdx.x / LPR, lane = threadIdx.x % LPR, idx = min(n, total - 1);
    const int tok = idx / d.kv_heads, g = idx - tok * d.kv_heads, pos = state[0] + tok;
    const bool mine = n < total && pos < d.capacity;
    const float* x = k + (size_t)tok * ldk + g * d.dimp;
    const size_t at = (size_t)g * d.capacity + pos;
    float ss = 0.0f;
    for (int i = lane * 4; i < d.dimp; i += LPR * 4) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(x + i);
#pragma unroll
        for (int e = 0; e < 4; e++) ss = fma_f(v[e], v[e], ss);
        if (!mine) continue;
        if constexpr (std::is_same<ET, float>::value) {
            *reinterpret_cast<f32x4*>(c.row + at * d.dimp + i) = v;
        } else {
            bf16x4 b;
#pragma unroll
            for (int e = 0; e < 4; e++) b[e] = (bf16_t)v[e];
            *reinterpret_cast<bf16x4*>(c.row + at * d.dimp + i) = b;
        }
    }
    ss = group_sum<LPR>(ss);
    if (lane == 0 && mine) c.inv_rms[at] = 1.0f / sqrtf(ss / (float)d.dim + d.eps);
}

template <typename ET>
int shared_kv_store(const SharedKvDims& d, const float* k, int ldk, SharedKvRows<ET> c, const int* state, int tokens, hipStream_t st) {
    FX_REQUIRE(k && c.row && c.inv_rms && state && tokens > 0 && ldk >= d.kv_heads * d.dimp && ldk % 4 == 0, "shared_kv_store: tokens=%d ldk=%d", tokens, ldk);
    const int total = tokens * d.kv_heads;
    if (d.dimp <= 64) shared_kv_store_kernel<ET, 16><<<(total + 15) / 16, 256, 0, st>>>(d, k, ldk, c, state, total);
    else if (d.dimp <= 128) shared_kv_store_kernel<ET, 32><<<(total + 7) / 8, 256, 0, st>>>(d, k, ldk, c, state, total);
    else shared_kv_store_kernel<ET, 64><<<(total + 3) / 4, 256, 0, st>>>(d, k, ldk, c, state, total);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int shared_kv_store<bf16_t>(const SharedKvDims&, const float*, int, SharedKvRows<bf16_t>, const int*, int, hipStream_t);
template int shared_kv_store<float>(const SharedKvDims&, const float*, int, SharedKvRows<float>, const int*, int, hipStream_t);

// ---- few tokens -----------------------------------------------------------------------------------------------------
constexpr int kKvSplits = 64, kKvStats = 4;               // most splits; floats behind a split's sums (maximum, weight sum)

static int kv_head_group(const SharedKvDims& d) {         // query heads per workgroup
    const int r = d.heads / d.kv_heads;
    return r >= 4 ? 4 : r >= 2 ? 2 : 1;
}
static int kv_split_count(const SharedKvDims& d) {
    const int gh = kv_head_group(d), blocks = d.kv_heads * ((d.heads / d.kv_heads + gh - 1) / gh);
    int s = 1;
    while (s < kKvSplits && s * blocks < 512) s *= 2;
    const int most = (d.capacity + 31) / 32;
    return s < most ? s : most;
}
size_t shared_kv_scratch(const SharedKvDims& d) { return (size_t)d.heads * kv_split_count(d) * (d.dimp + kKvStats); }

// N consecutive float32 (N a multiple of 4, 16-byte aligned), zeros where there are none.
template <int N>
__device__ __forceinline__ void load_floats(const float* p, bool there, float* v) {
#pragma unroll
    for (int i = 0; i < N / 4; i++) {
        const f32x4 u = there ? *reinterpret_cast<const f32x4*>(p + 4 * i) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int e = 0; e < 4; e++) v[4 * i + e] = u[e];
    }
}

// Rows per split when n rows are shared out over at most `splits`, and how many splits then have rows.
__device__ __forceinline__ int kv_split_rows(int n, int splits) { return max(((n + splits - 1) / splits + 31) / 32 * 32, 32); }
__device__ __forceinline__ int kv_splits_used(int n, int rows) { return max((n + rows - 1) / rows, 1); }

template <typename ET, int LPK, int GH, int CPL>
__global__ __launch_bounds__(256) void shared_kv_split_kernel(SharedKvDims d, const void* __restrict__ q, int ldq, int q_f32, const float* __restrict__ k, int ldk,
                                                              const float* __restrict__ norm_w, SharedKvRows<ET> c, const int* __restrict__ state, int tok0,
                                                              int splits, float* __restrict__ part) {
    constexpr int CE = Chunk<ET>::N, KS = 256 / LPK, U = 4, N = CPL * CE;
    extern __shared__ __attribute__((aligned(16))) float sums[];   // [4][GH][dimp]
    __shared__ float sm_m[4][GH], sm_l[4][GH];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, lc = lane % LPK, ks = wave * (64 / LPK) + lane / LPK;
    const int rep = d.heads / d.kv_heads, hb = (rep + GH - 1) / GH, g = blockIdx.y / hb, h0 = (blockIdx.y % hb) * GH, tok = blockIdx.z;
    const int base = state[0], pos = base + tok0 + tok, held = k ? base : pos + 1;      // rows 0 .. held-1 are in the cache
    const int per = kv_split_rows(held, splits), first = blockIdx.x * per, last = min(held, first + per);
    if ((int)blockIdx.x >= kv_splits_used(held, per) || pos >= d.capacity) return;
    const ET* rows = c.row + (size_t)g * d.capacity * d.dimp;
    const float* inv = c.inv_rms + (size_t)g * d.capacity;
    int col[CPL];
    bool in[CPL];
#pragma unroll
    for (int j = 0; j < CPL; j++) { col[j] = (lc + j * LPK) * CE; in[j] = col[j] < d.dimp; }

    auto load = [&](int b, i32x4 (&u)[U][CPL], float (&r)[U]) {
#pragma unroll
        for (int i = 0; i < U; i++) {
            const int key = min(first + (b * U + i) * KS + ks, last - 1);
#pragma unroll
            for (int j = 0; j < CPL; j++) u[i][j] = in[j] ? *reinterpret_cast<const i32x4*>(rows + (size_t)key * d.dimp + col[j]) : i32x4{0, 0, 0, 0};
            r[i] = inv[key];
        }
    };
    i32x4 ua[U][CPL], ub[U][CPL];
    float ra[U], rb[U];
    const int nb = last > first ? (last - first + U * KS - 1) / (U * KS) : 0;
    if (nb > 0) load(0, ua, ra);

    // ---- the queries' columns of this lane, normed and scaled
    float qv[GH][N];
    {
        float wv[N];
#pragma unroll
        for (int j = 0; j < CPL; j++) load_floats<CE>(norm_w + col[j], in[j], wv + j * CE);
        const float f = query_factor(d, pos);
#pragma unroll
        for (int h = 0; h < GH; h++) {
            const size_t at = (size_t)tok * ldq + (size_t)(g * rep + min(h0 + h, rep - 1)) * d.dimp;
            float ss = 0.0f;
#pragma unroll
            for (int j = 0; j < CPL; j++) {
                if (q_f32) {
                    load_floats<CE>(static_cast<const float*>(q) + at + col[j], in[j], &qv[h][j * CE]);
                } else {
                    uint4 u = make_uint4(0, 0, 0, 0);
                    if (in[j]) u = *reinterpret_cast<const uint4*>(static_cast<const ET*>(q) + at + col[j]);
                    Chunk<ET>::unpack(u, reinterpret_cast<float (&)[CE]>(qv[h][j * CE]));
                }
            }
#pragma unroll
            for (int e = 0; e < N; e++) ss = fma_f(qv[h][e], qv[h][e], ss);
            const float s = f / sqrtf(group_sum<LPK>(ss) / (float)d.dim + d.eps);
#pragma unroll
            for (int e = 0; e < N; e++) qv[h][e] *= s * wv[e];
        }
    }
    float m[GH], l[GH], acc[GH][N];
#pragma unroll
    for (int h = 0; h < GH; h++) {
        m[h] = -1e30f;                                    // finite, so that differences stay defined
        l[h] = 0.0f;
#pragma unroll
        for (int e = 0; e < N; e++) acc[h][e] = 0.0f;
    }
    // scores of one row's columns x, summed over the row's lanes
    auto score = [&](const float (&x)[N], int h) {
        float s = 0.0f;
#pragma unroll
        for (int e = 0; e < N; e++) s = fma_f(qv[h][e], x[e], s);
        return group_sum<LPK>(s);
    };
    auto take = [&](int b, const i32x4 (&u)[U][CPL], const float (&r)[U]) {
        float s[GH][U];
#pragma unroll
        for (int i = 0; i < U; i++) {
            float x[N];
#pragma unroll
            for (int j = 0; j < CPL; j++) Chunk<ET>::unpack(make_uint4(u[i][j][0], u[i][j][1], u[i][j][2], u[i][j][3]), reinterpret_cast<float (&)[CE]>(x[j * CE]));
            const bool seen = first + (b * U + i) * KS + ks < last;
#pragma unroll
            for (int h = 0; h < GH; h++) {
                const float v = score(x, h) * r[i];
                s[h][i] = seen ? v : -INFINITY;
            }
        }
#pragma unroll
        for (int h = 0; h < GH; h++) {
            float mx = m[h];
#pragma unroll
            for (int i = 0; i < U; i++) mx = fmaxf(mx, s[h][i]);
            const float al = __builtin_amdgcn_exp2f(m[h] - mx);
            m[h] = mx;
            l[h] *= al;
#pragma unroll
            for (int e = 0; e < N; e++) acc[h][e] *= al;
#pragma unroll
            for (int i = 0; i < U; i++) { s[h][i] = __builtin_amdgcn_exp2f(s[h][i] - mx); l[h] += s[h][i]; }
        }
#pragma unroll
        for (int i = 0; i < U; i++) {
            float x[N];
#pragma unroll
            for (int j = 0; j < CPL; j++) Chunk<ET>::unpack(make_uint4(u[i][j][0], u[i][j][1], u[i][j][2], u[i][j][3]), reinterpret_cast<float (&)[CE]>(x[j * CE]));
#pragma unroll
            for (int h = 0; h < GH; h++)
#pragma unroll
                for (int e = 0; e < N; e++) acc[h][e] = fma_f(s[h][i], x[e], acc[h][e]);
        }
    };
    for (int b = 0; b < nb; b += 2) {
        if (b + 1 < nb) load(b + 1, ub, rb);
        take(b, ua, ra);
        if (b + 1 >= nb) break;
        if (b + 2 < nb) load(b + 2, ua, ra);
        take(b + 1, ub, rb);
    }
    // ---- rows of this step, which are not in the cache yet: taken by the first split, stored by their own token
    if (k && blockIdx.x == 0) {
        for (int n0 = 0; n0 <= tok; n0 += KS) {
            const int n = min(n0 + ks, tok);
            const float* src = k + (size_t)n * ldk + g * d.dimp;
            float x[N], ss = 0.0f;
#pragma unroll
            for (int j = 0; j < CPL; j++) load_floats<CE>(src + col[j], in[j], x + j * CE);
#pragma unroll
            for (int e = 0; e < N; e++) {
                ss = fma_f(x[e], x[e], ss);
                x[e] = (float)(ET)x[e];                   // as a later step reads it
            }
            const float r = 1.0f / sqrtf(group_sum<LPK>(ss) / (float)d.dim + d.eps);
            const bool mine = n0 + ks <= tok;
            if (h0 == 0 && n0 + ks == tok) {
                const size_t at = (size_t)g * d.capacity + pos;
#pragma unroll
                for (int j = 0; j < CPL; j++)
                    if (in[j]) {
                        __attribute__((aligned(16))) ET o[CE];
#pragma unroll
                        for (int e = 0; e < CE; e++) o[e] = (ET)x[j * CE + e];
                        *reinterpret_cast<uint4*>(c.row + at * d.dimp + col[j]) = *reinterpret_cast<const uint4*>(o);
                    }
                if (lc == 0) c.inv_rms[at] = r;
            }
#pragma unroll
            for (int h = 0; h < GH; h++) {
                const float v = score(x, h) * r, s = mine ? v : -INFINITY;
                const float mx = fmaxf(m[h], s), al = __builtin_amdgcn_exp2f(m[h] - mx), p = __builtin_amdgcn_exp2f(s - mx);
                m[h] = mx;
                l[h] = l[h] * al + p;
#pragma unroll
                for (int e = 0; e < N; e++) acc[h][e] = fma_f(p, x[e], acc[h][e] * al);
            }
        }
    }
    // ---- the groups of lanes meet
    float mt[GH];
#pragma unroll
    for (int h = 0; h < GH; h++) {
        mt[h] = wave_max(m[h]);
        if (lane == 0) sm_m[wave][h] = mt[h];
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < GH; h++) {
        mt[h] = fmaxf(fmaxf(sm_m[0][h], sm_m[1][h]), fmaxf(sm_m[2][h], sm_m[3][h]));
        const float w = __builtin_amdgcn_exp2f(m[h] - mt[h]);
        const float lw = wave_sum(lc == 0 ? l[h] * w : 0.0f);
        if (lane == 0) sm_l[wave][h] = lw;
#pragma unroll
        for (int e = 0; e < N; e++) acc[h][e] *= w;
    }
    if constexpr (LPK < 64) {
        constexpr int R = GH * N, LEFT = R / (64 / LPK) > 0 ? R / (64 / LPK) : 1;
        static_assert((R & (R - 1)) == 0, "halves all the way");     // fewer values than groups: the last ones are held twice
        float* a = &acc[0][0];
        multi_sum_step<R, LPK>(a, lane);
        int r0 = 0;
#pragma unroll
        for (int mask = LPK, half = R / 2; mask < 64; mask *= 2, half /= 2)
            if (lane & mask) r0 += half;
#pragma unroll
        for (int i = 0; i < LEFT; i++) {
            const int v = r0 + i, h = v / N, e = v % N, cc = (lc + (e / CE) * LPK) * CE + e % CE;
            if (cc < d.dimp) sums[(wave * GH + h) * d.dimp + cc] = a[i];
        }
    } else {
#pragma unroll
        for (int h = 0; h < GH; h++)
#pragma unroll
            for (int j = 0; j < CPL; j++)
#pragma unroll
                for (int e = 0; e < CE; e++)
                    if (in[j]) sums[(wave * GH + h) * d.dimp + col[j] + e] = acc[h][j * CE + e];
    }
    __syncthreads();
    const int ld = d.dimp + kKvStats, step = GH * d.dimp;
    for (int i = t; i < step; i += 256) {
        const int h = i / d.dimp, e = i - h * d.dimp;
        if (h0 + h < rep)
            part[(((size_t)tok * d.heads + g * rep + h0 + h) * splits + blockIdx.x) * ld + e] = (sums[i] + sums[step + i]) + (sums[2 * step + i] + sums[3 * step + i]);
    }
    if (t < GH && h0 + t < rep) {
        float* o = part + (((size_t)tok * d.heads + g * rep + h0 + t) * splits + blockIdx.x) * ld + d.dimp;
        o[0] = fmaxf(fmaxf(sm_m[0][t], sm_m[1][t]), fmaxf(sm_m[2][t], sm_m[3][t]));
        o[1] = (sm_l[0][t] + sm_l[1][t]) + (sm_l[2][t] + sm_l[3][t]);
    }
}

// Join the splits of one (token, head); here the sink enters the sum of the weights.
template <typename OT>
__global__ __launch_bounds__(256) void shared_kv_join_kernel(SharedKvDims d, const float* __restrict__ part, const int* __restrict__ state, int tok0, int held_only,
                                                             int splits, OT* __restrict__ o, int ldo) {
    __shared__ float wsp[kKvSplits];
    __shared__ float sums[256];
    const int t = threadIdx.x, lane = t & 63, h = blockIdx.x, tok = blockIdx.y, ld = d.dimp + kKvStats;
    const int pos = state[0] + tok0 + tok, held = held_only ? state[0] : pos + 1;
    if (pos >= d.capacity) return;
    const int ns = kv_splits_used(held, kv_split_rows(held, splits));
    const float* p = part + ((size_t)tok * d.heads + h) * splits * ld;
    {
        const float ms = lane < ns ? p[lane * ld + d.dimp] : -1e30f, ls = lane < ns ? p[lane * ld + d.dimp + 1] : 0.0f;
        float m = wave_max(ms);
        if (d.sink) m = fmaxf(m, 0.0f);
        const float w = lane < ns ? __builtin_amdgcn_exp2f(ms - m) : 0.0f;
        float l = wave_sum(ls * w);
        if (d.sink) l += __builtin_amdgcn_exp2f(-m);
        if (t < 64) wsp[lane] = w / l;
    }
    __syncthreads();
    int width = 64;                                       // threads that share a split's columns
    while (width < d.dim && width < 256) width *= 2;
    const int parts = 256 / width, my = t / width;
    for (int c0 = 0; c0 < d.dim; c0 += width) {
        const int e = c0 + t % width;
        float v = 0.0f;
        if (e < d.dim)
#pragma unroll 16
            for (int s = my; s < ns; s += parts) v = fma_f(p[s * ld + e], wsp[s], v);
        sums[t] = v;
        __syncthreads();
        if (my == 0 && e < d.dim) {
            for (int i = 1; i < parts; i++) v += sums[i * width + t];
            o[(size_t)tok * ldo + h * d.dim + e] = (OT)v;
        }
        __syncthreads();
    }
}

template <typename ET, int LPK, int GH, int CPL>
static int launch_splits(const SharedKvDims& d, const void* q, int ldq, const float* k, int ldk, const float* norm_w, const SharedKvRows<ET>& c,
                         const int* state, int tok0, int tokens, float* scratch, int f32, hipStream_t st) {
    const int splits = kv_split_count(d), rep = d.heads / d.kv_heads;
    const dim3 grid(splits, d.kv_heads * ((rep + GH - 1) / GH), tokens);
    shared_kv_split_kernel<ET, LPK, GH, CPL><<<grid, 256, 4 * GH * d.dimp * sizeof(float), st>>>(d, q, ldq, f32, k, ldk, norm_w, c, state, tok0, splits, scratch);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

template <typename ET>
int shared_kv_splits(const SharedKvDims& d, const void* q, int ldq, const float* k, int ldk, const float* norm_w, SharedKvRows<ET> c, const int* state,
                     int tok0, int tokens, float* scratch, void* o, int ldo, int f32, hipStream_t st) {
    FX_REQUIRE(q && norm_w && c.row && c.inv_rms && state && scratch && o && tokens > 0 && (!k || tok0 == 0), "shared_kv_splits: null pointer, or %d tokens at %d", tokens, tok0);
    FX_REQUIRE(d.heads % d.kv_heads == 0 && d.dimp % 8 == 0 && d.dimp >= d.dim && d.dimp <= 512 && ldq % (f32 ? 4 : 8) == 0 && ldk % 4 == 0,
               "shared_kv_splits: %d heads on %d, rows of %d, strides %d %d", d.heads, d.kv_heads, d.dimp, ldq, ldk);
    const int chunks = d.dimp / Chunk<ET>::N, gh = kv_head_group(d);
    int rc;
#define FX_SPLITS(LPK, CPL)                                                                                                                \
    (gh == 4   ? launch_splits<ET, LPK, 4, CPL>(d, q, ldq, k, ldk, norm_w, c, state, tok0, tokens, scratch, f32, st)                    \
     : gh == 2 ? launch_splits<ET, LPK, 2, CPL>(d, q, ldq, k, ldk, norm_w, c, state, tok0, tokens, scratch, f32, st)                    \
               : launch_splits<ET, LPK, 1, CPL>(d, q, ldq, k, ldk, norm_w, c, state, tok0, tokens, scratch, f32, st))
    if (chunks <= 8) rc = FX_SPLITS(8, 1);
    else if (chunks <= 16) rc = FX_SPLITS(16, 1);
    else if (chunks <= 32) rc = FX_SPLITS(32, 1);
    else if (chunks <= 64) rc = FX_SPLITS(64, 1);
    else if constexpr (std::is_same<ET, float>::value) rc = FX_SPLITS(64, 2);
    else rc = FLEXLLM_EINVAL;                             // not reached: rows of 512 are 64 pieces
#undef FX_SPLITS
    if (rc) return rc;
    const int splits = kv_split_count(d);
    const dim3 grid(d.heads, tokens);
    if (f32) shared_kv_join_kernel<float><<<grid, 256, 0, st>>>(d, scratch, state, tok0, k != nullptr, splits, static_cast<float*>(o), ldo);
    else shared_kv_join_kernel<ET><<<grid, 256, 0, st>>>(d, scratch, state, tok0, k != nullptr, splits, static_cast<ET*>(o), ldo);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int shared_kv_splits<bf16_t>(const SharedKvDims&, const void*, int, const float*, int, const float*, SharedKvRows<bf16_t>, const int*, int, int, float*, void*, int, int, hipStream_t);
template int shared_kv_splits<float>(const SharedKvDims&, const void*, int, const float*, int, const float*, SharedKvRows<float>, const int*, int, int, float*, void*, int, int, hipStream_t);

// ---- many tokens ----------------------------------------------------------------------------------------------------
// Workgroup: NW waves x 32 queries over tiles of 64 rows.  The queries of a key/value head are numbered token by token, the
// heads that share the rows within a token (query n: token n / rep, head n % rep), so a tile of rows serves all of them.
// The score tile is formed transposed (rows x queries): a lane holds one query's scores, and its registers are already the
// operand of the second product, whose k slots are assigned to the rows in accumulator order (slot j of half-wave h = row
// 8 * (j / 4) + 4 * h + j % 4 of each 16), which the transposed reads follow.
// LDS: rows in planes of 8 columns [plane][64 rows][16 B], planes 64 B apart modulo the banks.  Planes beyond dimp repeat
// plane 0: they meet zeros on the query side, and their sums are not stored.
constexpr int kFlashRows = 64;

template <int DK, int NW>
__global__ __launch_bounds__(NW * 64, DK > 128 ? 1 : 2) void shared_kv_flash_kernel(SharedKvDims d, const bf16_t* __restrict__ q, int ldq, const float* __restrict__ norm_w,
                                                                                    SharedKvRows<bf16_t> c, int pos0, int tokens, bf16_t* __restrict__ o, int ldo) {
    constexpr int NP = DK / 8, KP = kFlashRows * 16 + 64, NVT = DK / 32, T = NW * 64, KCH = NP * kFlashRows / T;
    static_assert(KCH * T == NP * kFlashRows, "whole pieces per thread");
    using bf16x4v = __bf16 __attribute__((ext_vector_type(4)));
    __shared__ __attribute__((aligned(16))) int8_t lk[NP * KP];
    __shared__ __attribute__((aligned(16))) float lr[kFlashRows];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, half = lane >> 5, ln = lane & 31;
    const int rep = d.heads / d.kv_heads, total = tokens * rep;
    const int g = blockIdx.x % d.kv_heads, nq = gridDim.x / d.kv_heads;
    const int q0 = (nq - 1 - (int)blockIdx.x / d.kv_heads) * (NW * 32);  // the longest first
    const int wq0 = q0 + wave * 32, qn = min(wq0 + ln, total - 1), tok = qn / rep, head = g * rep + qn - tok * rep;
    const int qp = pos0 + tok;                            // this lane's position
    const int qmin = pos0 + min(wq0, total - 1) / rep, qmax = pos0 + min(wq0 + 31, total - 1) / rep;
    const int last = pos0 + (min(q0 + NW * 32, total) - 1) / rep;        // last row that the workgroup sees
    const bf16_t* rows = c.row + (size_t)g * d.capacity * d.dimp;
    const float* inv = c.inv_rms + (size_t)g * d.capacity;

    i32x4 rk[KCH];
    float rr = 0.0f;
    int koff[KCH];
#pragma unroll
    for (int i = 0; i < KCH; i++) koff[i] = ((t + T * i) % NP) * 8 < d.dimp ? ((t + T * i) % NP) * 8 : 0;
    auto load = [&](int kb) {
#pragma unroll
        for (int i = 0; i < KCH; i++) rk[i] = *reinterpret_cast<const i32x4*>(rows + (size_t)min(kb + (t + T * i) / NP, last) * d.dimp + koff[i]);
        if (t < kFlashRows) rr = inv[min(kb + t, last)];
    };
    load(0);
    // ---- the queries: norm, weights and scale in float32, then the products' operand
    bf16x8 fq[DK / 16];
    {
        const bf16_t* qh = q + (size_t)tok * ldq + (size_t)head * d.dimp;
        float ss = 0.0f;
#pragma unroll
        for (int s = 0; s < DK / 16; s++) {
            const int e0 = (s * 2 + half) * 8;
            uint4 u = make_uint4(0, 0, 0, 0);
            if (e0 < d.dimp) u = *reinterpret_cast<const uint4*>(qh + e0);
            fq[s] = *reinterpret_cast<const bf16x8*>(&u);
#pragma unroll
            for (int e = 0; e < 8; e++) ss = fma_f((float)fq[s][e], (float)fq[s][e], ss);
        }
        ss += lane_xor_f<32>(ss);
        const float f = query_factor(d, qp) / sqrtf(ss / (float)d.dim + d.eps);
#pragma unroll
        for (int s = 0; s < DK / 16; s++) {
            const int e0 = (s * 2 + half) * 8;
            if (e0 < d.dimp)
#pragma unroll
                for (int e = 0; e < 8; e++) fq[s][e] = (bf16_t)((float)fq[s][e] * (f * norm_w[e0 + e]));
        }
    }
    f32x16 acc[NVT];
#pragma unroll
    for (int i = 0; i < NVT; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) acc[i][r] = 0.0f;
    // of this lane's query; the sink is a score of 0 whose weight one half of the wave counts
    float m = d.sink ? 0.0f : -1e30f, l = d.sink && half == 0 ? 1.0f : 0.0f;
    // transposed read: of 16 lanes, lane n hands in the address of row n / 4, columns 4 (n % 4) .. +3 and gets column n of the 4 rows
    const int tl = lane & 15;
    const int tr0 = ((lane >> 4 & 1) * 2 + ((tl & 3) >> 1)) * KP + (half * 4 + (tl >> 2)) * 16 + (tl & 1) * 8;
    __attribute__((address_space(3))) int8_t* const lk3 = (__attribute__((address_space(3))) int8_t*)lk;

    for (int kb = 0; kb <= last; kb += kFlashRows) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < KCH; i++) *reinterpret_cast<i32x4*>(lk + ((t + T * i) % NP) * KP + ((t + T * i) / NP) * 16) = rk[i];
        if (t < kFlashRows) lr[t] = rr;
        __syncthreads();
        if (kb + kFlashRows <= last) load(kb + kFlashRows);
        if (kb > qmax) continue;
        f32x16 s[2];
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) s[j][r] = 0.0f;
#pragma unroll
        for (int st = 0; st < DK / 16; st++)
#pragma unroll
            for (int j = 0; j < 2; j++) {
                const bf16x8 fk = *reinterpret_cast<const bf16x8*>(lk + (st * 2 + half) * KP + (j * 32 + ln) * 16);
                s[j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fk, fq[st], s[j], 0, 0, 0);
            }
        float mx = m;
        const bool edge = kb + kFlashRows - 1 > qmin;     // the tile holds unseen rows
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int r4 = 0; r4 < 4; r4++) {
                const int row = j * 32 + r4 * 8 + half * 4;
                const f32x4 ir = *reinterpret_cast<const f32x4*>(lr + row);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    float v = s[j][r4 * 4 + e] * ir[e];
                    if (edge) v = kb + row + e <= qp ? v : -INFINITY;
                    s[j][r4 * 4 + e] = v;
                    mx = fmaxf(mx, v);
                }
            }
        mx = fmaxf(mx, lane_xor_f<32>(mx));
        const float al = __builtin_amdgcn_exp2f(m - mx);
        m = mx;
        if (__any(al != 1.0f)) {
#pragma unroll
            for (int i = 0; i < NVT; i++)
#pragma unroll
                for (int r = 0; r < 16; r++) acc[i][r] *= al;
        }
        float ls = 0.0f;
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const float p = __builtin_amdgcn_exp2f(s[j][r] - mx);
                s[j][r] = p;
                ls += p;
            }
        l = l * al + ls;
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int st = 0; st < 2; st++) {
                bf16x8 ph, pl;
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const float p = s[j][st * 8 + e];
                    const bf16_t hi = (bf16_t)p;
                    ph[e] = hi;
                    pl[e] = (bf16_t)(p - (float)hi);
                }
#pragma unroll
                for (int i = 0; i < NVT; i++) {
                    __attribute__((address_space(3))) int8_t* src = lk3 + tr0 + i * 4 * KP + (j * 32 + st * 16) * 16;
                    const bf16x4v a = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4v*)src);
                    const bf16x4v b = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4v*)(src + 8 * 16));
                    const bf16x8 fv = __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
                    acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fv, ph, acc[i], 0, 0, 0);
                    acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fv, pl, acc[i], 0, 0, 0);
                }
            }
    }
    l += lane_xor_f<32>(l);
    const float out = 1.0f / l;
    if (wq0 + ln < total) {
        bf16_t* dst = o + (size_t)tok * ldo + (size_t)head * d.dim;
        const bool vec = (d.dim & 3) == 0 && (ldo & 3) == 0;
#pragma unroll
        for (int i = 0; i < NVT; i++)
#pragma unroll
            for (int r4 = 0; r4 < 4; r4++) {
                const int v = i * 32 + r4 * 8 + half * 4;
                bf16x4 b;
#pragma unroll
                for (int e = 0; e < 4; e++) b[e] = (bf16_t)(acc[i][r4 * 4 + e] * out);
                if (vec) {
                    if (v < d.dim) *reinterpret_cast<bf16x4*>(dst + v) = b;
                } else {
#pragma unroll
                    for (int e = 0; e < 4; e++)
                        if (v + e < d.dim) dst[v + e] = b[e];
                }
            }
    }
}

bool shared_kv_flash_ok(const SharedKvDims& d) { return d.dimp <= 256; }
int shared_kv_flash(const SharedKvDims& d, const bf16_t* q, int ldq, const float* norm_w, SharedKvRows<bf16_t> c, int pos0, int tokens, bf16_t* o, int ldo,
                    hipStream_t st) {
    FX_REQUIRE(q && norm_w && c.row && c.inv_rms && o && tokens > 0 && shared_kv_flash_ok(d) && d.heads % d.kv_heads == 0 && d.dimp % 8 == 0 && d.dimp >= d.dim,
               "shared_kv_flash: %d heads on %d, rows of %d", d.heads, d.kv_heads, d.dimp);
    FX_REQUIRE(ldq % 8 == 0 && ldq >= d.heads * d.dimp && ldo >= d.heads * d.dim && pos0 >= 0 && pos0 + tokens <= d.capacity && (size_t)tokens * d.heads < (1u << 30),
               "shared_kv_flash: strides %d %d, %d tokens at %d of %d", ldq, ldo, tokens, pos0, d.capacity);
    const int total = tokens * (d.heads / d.kv_heads), g4 = (total + 127) / 128 * d.kv_heads, g2 = (total + 63) / 64 * d.kv_heads;
    // two waves per workgroup where four would leave CUs without one
#define FX_FLASH(DK)                                                                                                        \
    do {                                                                                                                    \
        if (DK > 128 || g4 >= 512) shared_kv_flash_kernel<DK, 4><<<g4, 256, 0, st>>>(d, q, ldq, norm_w, c, pos0, tokens, o, ldo);       \
        else shared_kv_flash_kernel<(DK > 128 ? 128 : DK), 2><<<g2, 128, 0, st>>>(d, q, ldq, norm_w, c, pos0, tokens, o, ldo);                 \
    } while (0)
    if (d.dimp <= 64) FX_FLASH(64);
    else if (d.dimp <= 128) FX_FLASH(128);
    else FX_FLASH(256);
#undef FX_FLASH
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

}  // namespace fx
