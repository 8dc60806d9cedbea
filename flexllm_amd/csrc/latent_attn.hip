// Latent attention: a token leaves one normed latent and one rotated key part, shared by all heads, in the cache.
//
// Few tokens: the unrotated query goes through W_uk into the latent space and attends over the cached rows themselves,
// so a key costs its latent once for all of its per-head forms; the context comes back through W_uv.  Three kernels:
// carry the query over, attend over splits of the visible keys, join the splits and project.
// Many tokens: per-head keys and (transposed) values are formed once by two GEMMs over the visible rows, and a
// flash-style kernel runs on v_mfma_f32_32x32x16_bf16.  Scores and weights are float32 throughout: the weights enter the
// second product as the sum of two bfloat16 halves, which keeps 16 bits of each.
#include "float_ops.h"

namespace fx {

// ---- rows of a step into the cache, rotation of the queries -----------------------------------------------------
template <typename ET>
__global__ __launch_bounds__(256) void latent_store_kernel(LatentDims d, ET* __restrict__ q, int ldq, const float* __restrict__ raw, int ld_raw,
                                                           const float* __restrict__ norm_w, const float* __restrict__ cos_t,
                                                           const float* __restrict__ sin_t, ET* __restrict__ cache, const int* __restrict__ state) {
    __shared__ float red[4];
    const int t = threadIdx.x, tok = blockIdx.x, pos = state[0] + tok, rh = d.rot_dim >> 1;
    if (pos >= d.capacity) return;
    const float* cs = cos_t + (size_t)pos * rh;
    const float* sn = sin_t + (size_t)pos * rh;
    if (raw) {
        const float* x = raw + (size_t)tok * ld_raw;
        ET* row = cache + (size_t)pos * d.ldc;
        float ss = 0.0f;
        for (int i = t; i < d.kv_rank; i += 256) ss = fma_f(x[i], x[i], ss);
        const float rs = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)d.kv_rank + d.eps);
        for (int i = t; i < d.kv_rank; i += 256) row[i] = (ET)(x[i] * rs * norm_w[i]);
        for (int i = t; i < rh; i += 256) {
            const float u = x[d.kv_rank + 2 * i], v = x[d.kv_rank + 2 * i + 1];
            row[d.kvp + 2 * i] = (ET)(u * cs[i] - v * sn[i]);
            row[d.kvp + 2 * i + 1] = (ET)(v * cs[i] + u * sn[i]);
        }
    }
    ET* qr = q + (size_t)tok * ldq;
    const int step = d.dim + d.rot_dim;
    for (int i = t; i < d.heads * rh; i += 256) {
        const int h = i / rh, j = i - h * rh;
        ET* p = qr + h * step + d.dim + 2 * j;
        const float u = (float)p[0], v = (float)p[1];
        p[0] = (ET)(u * cs[j] - v * sn[j]);
        p[1] = (ET)(v * cs[j] + u * sn[j]);
    }
}

template <typename ET>
int latent_store(const LatentDims& d, ET* q, int ldq, const float* raw, int ld_raw, const float* norm_w, const float* cos_t,
                 const float* sin_t, ET* cache, const int* state, int tokens, hipStream_t st) {
    FX_REQUIRE(q && cos_t && sin_t && state && tokens > 0 && (!raw || (cache && norm_w)), "latent_store: null pointer");
    latent_store_kernel<ET><<<tokens, 256, 0, st>>>(d, q, ldq, raw, ld_raw, norm_w, cos_t, sin_t, cache, state);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int latent_store<bf16_t>(const LatentDims&, bf16_t*, int, const float*, int, const float*, const float*, const float*, bf16_t*, const int*, int, hipStream_t);
template int latent_store<float>(const LatentDims&, float*, int, const float*, int, const float*, const float*, const float*, float*, const int*, int, hipStream_t);

// ---- attention in the latent space --------------------------------------------------------------------------------
constexpr int kAbsCols = 128;                             // latent columns per workgroup of the query kernel
constexpr int kMaxSplits = 32;

struct LatentSplits { int keys, count; };                 // keys per split (a multiple of 64), splits per (token, head)
static LatentSplits latent_splits(const LatentDims& d) {
    const int most = d.window > 0 && d.window < d.capacity ? d.window : d.capacity;
    LatentSplits s;
    s.keys = ((most + kMaxSplits - 1) / kMaxSplits + 63) / 64 * 64;
    s.count = (most + s.keys - 1) / s.keys;
    return s;
}
size_t latent_absorbed_scratch(const LatentDims& d) {
    return (size_t)d.heads * d.ldc + (size_t)d.heads * latent_splits(d).count * (d.kvp + 2);
}

template <typename ET>
__global__ __launch_bounds__(256) void latent_query_kernel(LatentDims d, const ET* __restrict__ q, int ldq, const ET* __restrict__ w_uk,
                                                           float* __restrict__ ql, int slices) {
    constexpr int CE = Chunk<ET>::N, NC = kAbsCols / CE, NG = 256 / NC;
    __shared__ float part[NG][kAbsCols];
    const int t = threadIdx.x, h = blockIdx.x / slices, c0 = (blockIdx.x % slices) * kAbsCols, tok = blockIdx.y;
    const ET* qh = q + (size_t)tok * ldq + h * (d.dim + d.rot_dim);
    float* out = ql + ((size_t)tok * d.heads + h) * d.ldc;
    const int c = t % NC, g = t / NC, col = c0 + c * CE;
    float acc[CE];
#pragma unroll
    for (int e = 0; e < CE; e++) acc[e] = 0.0f;
    if (col < d.kvp) {
#pragma unroll 8
        for (int i = g; i < d.dim; i += NG) {
            const uint4 u = *reinterpret_cast<const uint4*>(w_uk + ((size_t)h * d.dim + i) * d.kvp + col);
            float wv[CE];
            Chunk<ET>::unpack(u, wv);
            const float qv = (float)qh[i];
#pragma unroll
            for (int e = 0; e < CE; e++) acc[e] = fma_f(wv[e], qv, acc[e]);
        }
    }
#pragma unroll
    for (int e = 0; e < CE; e++) part[g][c * CE + e] = acc[e];
    __syncthreads();
    if (t < kAbsCols && c0 + t < d.kvp) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < NG; i++) s += part[i][t];
        out[c0 + t] = s;
    }
    if (blockIdx.x % slices == 0)
        for (int i = t; i < d.ldc - d.kvp; i += 256) out[d.kvp + i] = i < d.rot_dim ? (float)qh[d.dim + i] : 0.0f;
}

// The query kernel of a decode step, which also leaves the tokens' own rows in the cache: workgroups 0 .. heads * slices - 1
// carry the queries over (rotating their rotated part on the way), the last one stores the row.
template <typename ET>
__global__ __launch_bounds__(256) void latent_store_query_kernel(LatentDims d, const float* __restrict__ q, int ldq, const float* __restrict__ raw, int ld_raw,
                                                                 const float* __restrict__ norm_w, const float* __restrict__ cos_t,
                                                                 const float* __restrict__ sin_t, ET* __restrict__ cache, const int* __restrict__ state,
                                                                 const ET* __restrict__ w_uk, float* __restrict__ ql, int slices) {
    constexpr int CE = Chunk<ET>::N, NC = kAbsCols / CE, NG = 256 / NC;
    __shared__ float part[NG][kAbsCols];
    __shared__ float red[4];
    const int t = threadIdx.x, tok = blockIdx.y, rh = d.rot_dim >> 1;
    const int h = blockIdx.x / slices, slice = blockIdx.x % slices;
    if (h == d.heads) {
        const int pos = state[0] + tok;
        if (!raw || pos >= d.capacity) return;
        const float* x = raw + (size_t)tok * ld_raw;
        ET* row = cache + (size_t)pos * d.ldc;
        float ss = 0.0f;
        for (int i = t; i < d.kv_rank; i += 256) ss = fma_f(x[i], x[i], ss);
        const float rs = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)d.kv_rank + d.eps);
        for (int i = t; i < d.kv_rank; i += 256) row[i] = (ET)(x[i] * rs * norm_w[i]);
        for (int i = t; i < rh; i += 256) {
            const float u = x[d.kv_rank + 2 * i], v = x[d.kv_rank + 2 * i + 1], c = cos_t[(size_t)pos * rh + i], s = sin_t[(size_t)pos * rh + i];
            row[d.kvp + 2 * i] = (ET)(u * c - v * s);
            row[d.kvp + 2 * i + 1] = (ET)(v * c + u * s);
        }
        return;
    }
    const float* qh = q + (size_t)tok * ldq + h * (d.dim + d.rot_dim);
    float* out = ql + ((size_t)tok * d.heads + h) * d.ldc;
    const int c = t % NC, g = t / NC, c0 = slice * kAbsCols, col = c0 + c * CE;
    float acc[CE];
#pragma unroll
    for (int e = 0; e < CE; e++) acc[e] = 0.0f;
    if (col < d.kvp) {
#pragma unroll 8
        for (int i = g; i < d.dim; i += NG) {
            const uint4 u = *reinterpret_cast<const uint4*>(w_uk + ((size_t)h * d.dim + i) * d.kvp + col);
            float wv[CE];
            Chunk<ET>::unpack(u, wv);
            const float qv = qh[i];
#pragma unroll
            for (int e = 0; e < CE; e++) acc[e] = fma_f(wv[e], qv, acc[e]);
        }
    }
#pragma unroll
    for (int e = 0; e < CE; e++) part[g][c * CE + e] = acc[e];
    __syncthreads();
    if (t < kAbsCols && c0 + t < d.kvp) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < NG; i++) s += part[i][t];
        out[c0 + t] = s;
    }
    if (slice == 0) {
        const int pos = min(state[0] + tok, d.capacity - 1);
        for (int i = t; i < d.ldc - d.kvp; i += 256) {
            float v = 0.0f;
            if (i < d.rot_dim) {
                const int j = i >> 1;
                const float a = qh[d.dim + 2 * j], b = qh[d.dim + 2 * j + 1], cs = cos_t[(size_t)pos * rh + j], sn = sin_t[(size_t)pos * rh + j];
                v = i & 1 ? b * cs + a * sn : a * cs - b * sn;
            }
            out[d.kvp + i] = v;
        }
    }
}

// One split of the visible keys of one (token, head): scores, their maximum and sum, and the weighted sum of latents.
template <typename ET>
__global__ __launch_bounds__(256) void latent_split_kernel(LatentDims d, const float* __restrict__ ql, const ET* __restrict__ cache,
                                                           const int* __restrict__ state, int tok0, int keys, int splits, float* __restrict__ part) {
    constexpr int CE = Chunk<ET>::N;
    extern __shared__ __attribute__((aligned(16))) float sm[];     // q [ldc], scores [keys], sums [256 * CE]
    __shared__ float red[4];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, h = blockIdx.y, tok = blockIdx.z;
    const int pos = state[0] + tok0 + tok;
    const int lo = d.window > 0 && pos - d.window + 1 > 0 ? pos - d.window + 1 : 0;
    const int first = lo + blockIdx.x * keys, n = min(keys, pos + 1 - first);
    if (n <= 0 || pos >= d.capacity) return;
    float *sq = sm, *sc = sm + d.ldc, *sum = sc + keys;
    const float* qv = ql + ((size_t)tok * d.heads + h) * d.ldc;
    for (int i = t; i < d.ldc; i += 256) sq[i] = qv[i];
    __syncthreads();
    const ET* base = cache + (size_t)first * d.ldc;
    const int nch = d.ldc / CE;
    float mx = -INFINITY;
    constexpr int KW = 8;                                 // keys of a wave in flight
    for (int k0 = wave * KW; k0 < n; k0 += 4 * KW) {
        float acc[KW] = {0, 0, 0, 0, 0, 0, 0, 0};
        for (int c = lane; c < nch; c += 64) {
            uint4 u[KW];
#pragma unroll
            for (int i = 0; i < KW; i++) u[i] = *reinterpret_cast<const uint4*>(base + (size_t)min(k0 + i, n - 1) * d.ldc + c * CE);
            float x[CE];
#pragma unroll
            for (int e = 0; e < CE; e++) x[e] = sq[c * CE + e];
#pragma unroll
            for (int i = 0; i < KW; i++) {
                float kv[CE];
                Chunk<ET>::unpack(u[i], kv);
#pragma unroll
                for (int e = 0; e < CE; e++) acc[i] = fma_f(kv[e], x[e], acc[i]);
            }
        }
        multi_sum_step<KW, 1>(acc, lane);
        if (lane < KW) {
            const int k = k0 + multi_row<KW>(lane);
            const float s = acc[0] * d.scale;
            if (k < n) { sc[k] = s; mx = fmaxf(mx, s); }
        }
    }
    mx = block_max<4>(mx, red);
    float l = 0.0f;
    for (int i = t; i < n; i += 256) { const float p = exp_f<false>(sc[i] - mx); sc[i] = p; l += p; }
    l = block_sum<4>(l, red);                             // its barriers also publish the weights
    float* out = part + (((size_t)tok * d.heads + h) * splits + blockIdx.x) * (d.kvp + 2);
    if (t == 0) { out[d.kvp] = mx; out[d.kvp + 1] = l; }
    const int ncl = d.kvp / CE;
    for (int cb = 0; cb < ncl; cb += 256) {
        const int nc = min(256, ncl - cb), groups = 256 / nc, c = t % nc, g = t / nc;
        float acc[CE];
#pragma unroll
        for (int e = 0; e < CE; e++) acc[e] = 0.0f;
        if (g < groups) {
#pragma unroll 8
            for (int k = g; k < n; k += groups) {
                float kv[CE];
                Chunk<ET>::unpack(*reinterpret_cast<const uint4*>(base + (size_t)k * d.ldc + (cb + c) * CE), kv);
                const float p = sc[k];
#pragma unroll
                for (int e = 0; e < CE; e++) acc[e] = fma_f(p, kv[e], acc[e]);
            }
#pragma unroll
            for (int e = 0; e < CE; e++) sum[(g * nc + c) * CE + e] = acc[e];
        }
        __syncthreads();
        for (int i = t; i < nc * CE; i += 256) {
            float s = 0.0f;
            for (int j = 0; j < groups; j++) s += sum[j * nc * CE + i];
            out[cb * CE + i] = s;
        }
        __syncthreads();
    }
}

// The same with the split's rows staged in LDS, tile by tile (TK rows), so that the cache is read in one burst per tile and
// both passes over a tile run from LDS; sums of earlier tiles are rescaled as the maximum grows.  A thread owns the latent
// columns of piece t % ncl for every G-th row.
constexpr int kSplitPieces = 20;                          // 16-byte pieces in flight per thread
template <typename ET>
__global__ __launch_bounds__(256) void latent_split_tile_kernel(LatentDims d, const float* __restrict__ ql, const ET* __restrict__ cache,
                                                                const int* __restrict__ state, int tok0, int keys, int splits, int tk, float* __restrict__ part) {
    constexpr int CE = Chunk<ET>::N, KW = 4;
    extern __shared__ __attribute__((aligned(16))) int8_t sm8[];   // rows [tk][ldc] of ET, q [ldc], weights [tk], sums [256 * CE]
    __shared__ float red[4];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, h = blockIdx.y, tok = blockIdx.z;
    ET* rows = reinterpret_cast<ET*>(sm8);
    float* sq = reinterpret_cast<float*>(sm8 + (size_t)tk * d.ldc * sizeof(ET));
    float *sc = sq + d.ldc, *sum = sc + tk;
    const float* qv = ql + ((size_t)tok * d.heads + h) * d.ldc;
    const int pos = state[0] + tok0 + tok;
    const int lo = d.window > 0 && pos - d.window + 1 > 0 ? pos - d.window + 1 : 0;
    const int first = lo + blockIdx.x * keys, n = min(keys, pos + 1 - first);
    if (n <= 0 || pos >= d.capacity) return;
    const int nch = d.ldc / CE, ncl = d.kvp / CE, groups = 256 / ncl, c = t % ncl, g = t / ncl;
    float m = -INFINITY, l = 0.0f, acc[CE];
#pragma unroll
    for (int e = 0; e < CE; e++) acc[e] = 0.0f;
    for (int k0 = 0; k0 < n; k0 += tk) {
        const int nk = min(tk, n - k0), total = nk * nch;
        const i32x4* src = reinterpret_cast<const i32x4*>(cache + (size_t)(first + k0) * d.ldc);    // the rows are one run of memory
        i32x4* dst = reinterpret_cast<i32x4*>(rows);
        __syncthreads();                                  // the previous tile has been read
        for (int b = 0; b < total; b += 256 * kSplitPieces) {
            i32x4 u[kSplitPieces];
#pragma unroll
            for (int i = 0; i < kSplitPieces; i++) u[i] = src[min(b + 256 * i + t, total - 1)];
            if (k0 == 0 && b == 0)                        // the query follows the first rows on their way
                for (int i = t; i < d.ldc; i += 256) sq[i] = qv[i];
#pragma unroll
            for (int i = 0; i < kSplitPieces; i++)
                if (b + 256 * i + t < total) dst[b + 256 * i + t] = u[i];
        }
        __syncthreads();
        float mx = -INFINITY;
        for (int k = wave * KW; k < nk; k += 4 * KW) {
            float a[KW] = {0, 0, 0, 0};
            for (int cc = lane; cc < nch; cc += 64) {
                float x[CE];
#pragma unroll
                for (int q4 = 0; q4 < CE / 4; q4++) {
                    const f32x4 v = *reinterpret_cast<const f32x4*>(sq + cc * CE + q4 * 4);
#pragma unroll
                    for (int e = 0; e < 4; e++) x[q4 * 4 + e] = v[e];
                }
#pragma unroll
                for (int i = 0; i < KW; i++) {
                    float kv[CE];
                    Chunk<ET>::unpack(*reinterpret_cast<const uint4*>(rows + (size_t)min(k + i, nk - 1) * d.ldc + cc * CE), kv);
#pragma unroll
                    for (int e = 0; e < CE; e++) a[i] = fma_f(kv[e], x[e], a[i]);
                }
            }
            multi_sum_step<KW, 1>(a, lane);
            if (lane < KW) {
                const int key = k + multi_row<KW>(lane);
                const float s = a[0] * d.scale;
                if (key < nk) { sc[key] = s; mx = fmaxf(mx, s); }
            }
        }
        mx = fmaxf(m, block_max<4>(mx, red));
        const float al = k0 == 0 ? 0.0f : exp_f<false>(m - mx);
        m = mx;
        float ls = 0.0f;
        if (t < nk) { const float p = exp_f<false>(sc[t] - mx); sc[t] = p; ls = p; }
        l = l * al + block_sum<4>(ls, red);
#pragma unroll
        for (int e = 0; e < CE; e++) acc[e] *= al;
        if (g < groups)
#pragma unroll 4
            for (int k = g; k < nk; k += groups) {
                float kv[CE];
                Chunk<ET>::unpack(*reinterpret_cast<const uint4*>(rows + (size_t)k * d.ldc + c * CE), kv);
                const float p = sc[k];
#pragma unroll
                for (int e = 0; e < CE; e++) acc[e] = fma_f(p, kv[e], acc[e]);
            }
    }
    float* out = part + (((size_t)tok * d.heads + h) * splits + blockIdx.x) * (d.kvp + 2);
    if (t == 0) { out[d.kvp] = m; out[d.kvp + 1] = l; }
    if (g < groups)
#pragma unroll
        for (int e = 0; e < CE; e++) sum[(g * ncl + c) * CE + e] = acc[e];
    __syncthreads();
    for (int i = t; i < d.kvp; i += 256) {
        float s = 0.0f;
        for (int j = 0; j < groups; j++) s += sum[j * d.kvp + i];
        out[i] = s;
    }
}

// Join the splits of one (token, head) and carry the context back: 32 value rows per workgroup.
template <typename ET, typename OT>
__global__ __launch_bounds__(256) void latent_join_kernel(LatentDims d, const float* __restrict__ part, const ET* __restrict__ w_uv,
                                                          const int* __restrict__ state, int tok0, int keys, int splits, int slices,
                                                          OT* __restrict__ o, int ldo) {
    constexpr int CE = Chunk<ET>::N;
    extern __shared__ __attribute__((aligned(16))) float ctx[];
    __shared__ float wsp[64];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, h = blockIdx.x / slices, v0 = (blockIdx.x % slices) * 32, tok = blockIdx.y;
    const int pos = state[0] + tok0 + tok;
    if (pos >= d.capacity) return;
    const int vis = d.window > 0 ? min(pos + 1, d.window) : pos + 1, ns = (vis + keys - 1) / keys;
    const float* p = part + ((size_t)tok * d.heads + h) * splits * (d.kvp + 2);
    const int ld = d.kvp + 2;
    const int nch = d.kvp / CE, r0 = v0 + wave * 8;
    auto rows = [&](int c, uint4 (&u)[8]) {
#pragma unroll
        for (int i = 0; i < 8; i++) u[i] = *reinterpret_cast<const uint4*>(w_uv + ((size_t)h * d.vdim + min(r0 + i, d.vdim - 1)) * d.kvp + c * CE);
    };
    uint4 first[8];                                       // requested before the splits are joined
    rows(min(lane, nch - 1), first);
    {
        // every wave forms the splits' weights, a lane per split (there are at most kMaxSplits <= 64)
        const float ms = lane < ns ? p[lane * ld + d.kvp] : -INFINITY, ls = lane < ns ? p[lane * ld + d.kvp + 1] : 0.0f;
        const float m = wave_max(ms);
        const float w = lane < ns ? exp_f<false>(ms - m) : 0.0f;
        const float l = wave_sum(ls * w);
        if (wave == 0) wsp[lane] = w / l;
    }
    __syncthreads();
    for (int i = t; i < d.kvp; i += 256) {
        float c = 0.0f;
#pragma unroll 8
        for (int s = 0; s < ns; s++) c = fma_f(p[s * ld + i], wsp[s], c);
        ctx[i] = c;
    }
    __syncthreads();
    float acc[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    for (int c = lane; c < nch; c += 64) {
        uint4 u[8];
        if (c == lane) {
#pragma unroll
            for (int i = 0; i < 8; i++) u[i] = first[i];
        } else {
            rows(c, u);
        }
        float x[CE];
#pragma unroll
        for (int e = 0; e < CE; e++) x[e] = ctx[c * CE + e];
#pragma unroll
        for (int i = 0; i < 8; i++) {
            float wv[CE];
            Chunk<ET>::unpack(u[i], wv);
#pragma unroll
            for (int e = 0; e < CE; e++) acc[i] = fma_f(wv[e], x[e], acc[i]);
        }
    }
    multi_sum_step<8, 1>(acc, lane);
    if (lane < 8) {
        const int v = r0 + multi_row<8>(lane);
        if (v < d.vdim) o[(size_t)tok * ldo + h * d.vdim + v] = (OT)acc[0];
    }
}

template <typename ET>
static int latent_attend(const LatentDims& d, const float* ql, float* part, const ET* w_uv, const ET* cache, const int* state, int tok0, int tokens,
                         void* o, int ldo, int o_f32, hipStream_t st) {
    const LatentSplits sp = latent_splits(d);
    size_t lds = (size_t)(d.ldc + sp.keys + 256 * Chunk<ET>::N) * sizeof(float);
    FX_REQUIRE(lds <= 60 * 1024 && d.kvp * sizeof(float) <= 60 * 1024, "latent_absorbed: latent of %d (padded) with %d keys per split exceeds LDS", d.kvp, sp.keys);
    int tk = 64;                                          // rows per tile: at most 76 KiB, two workgroups per CU
    while (tk > 8 && (size_t)tk * d.ldc * sizeof(ET) > 76 * 1024) tk /= 2;
    if (d.kvp <= 256 * Chunk<ET>::N && (size_t)tk * d.ldc * sizeof(ET) <= 76 * 1024) {
        lds = (size_t)tk * d.ldc * sizeof(ET) + (size_t)(d.ldc + tk + 256 * Chunk<ET>::N) * sizeof(float);
        FX_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(latent_split_tile_kernel<ET>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        latent_split_tile_kernel<ET><<<dim3(sp.count, d.heads, tokens), 256, lds, st>>>(d, ql, cache, state, tok0, sp.keys, sp.count, tk, part);
    } else {
        latent_split_kernel<ET><<<dim3(sp.count, d.heads, tokens), 256, lds, st>>>(d, ql, cache, state, tok0, sp.keys, sp.count, part);
    }
    const int vs = (d.vdim + 31) / 32;
    if (o_f32) latent_join_kernel<ET, float><<<dim3(d.heads * vs, tokens), 256, d.kvp * sizeof(float), st>>>(d, part, w_uv, state, tok0, sp.keys, sp.count, vs, static_cast<float*>(o), ldo);
    else latent_join_kernel<ET, ET><<<dim3(d.heads * vs, tokens), 256, d.kvp * sizeof(float), st>>>(d, part, w_uv, state, tok0, sp.keys, sp.count, vs, static_cast<ET*>(o), ldo);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

template <typename ET>
int latent_absorbed(const LatentDims& d, const ET* q, int ldq, const ET* w_uk, const ET* w_uv, const ET* cache, const int* state,
                    int tok0, int tokens, float* scratch, ET* o, int ldo, hipStream_t st) {
    FX_REQUIRE(q && w_uk && w_uv && cache && state && scratch && o && tokens > 0, "latent_absorbed: null pointer");
    const int slices = (d.kvp + kAbsCols - 1) / kAbsCols;
    latent_query_kernel<ET><<<dim3(d.heads * slices, tokens), 256, 0, st>>>(d, q, ldq, w_uk, scratch, slices);
    return latent_attend<ET>(d, scratch, scratch + (size_t)tokens * d.heads * d.ldc, w_uv, cache, state, tok0, tokens, o, ldo, 0, st);
}
template int latent_absorbed<bf16_t>(const LatentDims&, const bf16_t*, int, const bf16_t*, const bf16_t*, const bf16_t*, const int*, int, int, float*, bf16_t*, int, hipStream_t);
template int latent_absorbed<float>(const LatentDims&, const float*, int, const float*, const float*, const float*, const int*, int, int, float*, float*, int, hipStream_t);

template <typename ET>
int latent_decode(const LatentDims& d, const float* q, int ldq, const float* raw, int ld_raw, const float* norm_w, const float* cos_t, const float* sin_t,
                  const ET* w_uk, const ET* w_uv, ET* cache, const int* state, int tokens, float* scratch, float* o, int ldo, hipStream_t st) {
    FX_REQUIRE(q && cos_t && sin_t && w_uk && w_uv && cache && state && scratch && o && tokens > 0 && (!raw || norm_w), "latent_decode: null pointer");
    const int slices = (d.kvp + kAbsCols - 1) / kAbsCols;
    latent_store_query_kernel<ET><<<dim3(d.heads * slices + 1, tokens), 256, 0, st>>>(d, q, ldq, raw, ld_raw, norm_w, cos_t, sin_t, cache, state, w_uk, scratch, slices);
    return latent_attend<ET>(d, scratch, scratch + (size_t)tokens * d.heads * d.ldc, w_uv, cache, state, 0, tokens, o, ldo, 1, st);
}
template int latent_decode<bf16_t>(const LatentDims&, const float*, int, const float*, int, const float*, const float*, const float*, const bf16_t*, const bf16_t*, bf16_t*, const int*, int, float*, float*, int, hipStream_t);
template int latent_decode<float>(const LatentDims&, const float*, int, const float*, int, const float*, const float*, const float*, const float*, const float*, float*, const int*, int, float*, float*, int, hipStream_t);

// ---- attention of many tokens --------------------------------------------------------------------------------------
// Workgroup: NW waves x 32 queries of one head over key tiles of 64.  The score tile is formed transposed (keys x
// queries), so that a lane holds one query's scores, and its registers are already the operand of the second product:
// the slots of that product's k dimension are assigned to the keys in accumulator order (slot j of half-wave h = key
// 8 * (j / 4) + 4 * h + j % 4 of each 16), which the reads of the transposed values follow.
// LDS: keys in planes of 8 dims [plane][64 keys][16 B], values in planes of 4 keys [plane][value row][8 B].
// Planes beyond a head's own dims meet zeros on the query side, value rows beyond vdim are not stored: both may hold any
// finite value, so no load is conditional.
constexpr int kFlashK = 64;

template <int DK, int DV, int NW>
__global__ __launch_bounds__(NW * 64, (DV > 128 || NW < 4) ? 1 : 2) void latent_flash_kernel(LatentDims d, const bf16_t* __restrict__ q, int ldq, const bf16_t* __restrict__ k, int ldk,
                                                           const bf16_t* __restrict__ vt, int ldv, const bf16_t* __restrict__ cache, int kv0, int pos0,
                                                           int tokens, int rows, bf16_t* __restrict__ o, int ldo) {
    constexpr int NP = DK / 8, KP = kFlashK * 16 + 32, VP = DV * 8 + 16, NVT = DV / 32;
    constexpr int T = NW * 64, kFlashQ = NW * 32;
    constexpr int KCH = NP * kFlashK / T, VCH = DV * 8 / T;              // 16-byte pieces per thread and tile
    __shared__ __attribute__((aligned(16))) int8_t lk[NP * KP];
    __shared__ __attribute__((aligned(16))) int8_t lv[16 * VP];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, half = lane >> 5, ln = lane & 31;
    const int h = blockIdx.x % d.heads, q0 = (blockIdx.x / d.heads) * kFlashQ;
    const int dim8 = (d.dim + 15) / 16 * 2;                              // planes of the unrotated part (padded)
    const int wq0 = q0 + wave * 32, qi = min(wq0 + ln, tokens - 1);
    const uint4 zero = make_uint4(0, 0, 0, 0);

    bf16x8 fq[DK / 16];
    const bf16_t* qh = q + (size_t)qi * ldq + h * (d.dim + d.rot_dim);
#pragma unroll
    for (int s = 0; s < DK / 16; s++) {
        const int pl = s * 2 + half;
        uint4 u = zero;
        if (pl < dim8) { if (pl * 8 < d.dim) u = *reinterpret_cast<const uint4*>(qh + pl * 8); }
        else if ((pl - dim8) * 8 < d.rot_dim) u = *reinterpret_cast<const uint4*>(qh + d.dim + (pl - dim8) * 8);
        fq[s] = *reinterpret_cast<const bf16x8*>(&u);
    }
    f32x16 acc[NVT];
#pragma unroll
    for (int i = 0; i < NVT; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) acc[i][r] = 0.0f;
    float m = -1e30f, l = 0.0f;                           // of this lane's query; m finite so that differences stay defined
    const float sc2 = d.scale * 1.44269504088896340736f;

    const int last_q = min(q0 + kFlashQ, tokens) - 1;
    const int lo_pos = d.window > 0 ? max(0, pos0 + q0 - d.window + 1) : 0;
    const int kb0 = max(0, lo_pos - kv0) / kFlashK * kFlashK, kb1 = pos0 + last_q - kv0;
    const int qp = pos0 + wq0 + ln;                       // this lane's position
    const int qmin = pos0 + wq0, qmax = pos0 + wq0 + 31;

    i32x4 rk[KCH], rv[VCH];
    const bf16_t* kbase[KCH];                             // row 0 of the piece's source, its row and row length
    int krow[KCH], kld[KCH], voff[VCH];
#pragma unroll
    for (int i = 0; i < KCH; i++) {
        const int c = t + T * i, pl = c % NP;
        const bool rot = pl >= dim8 && (pl - dim8) * 8 < d.rot_dim;
        kbase[i] = rot ? cache + (size_t)kv0 * d.ldc + d.kvp + (pl - dim8) * 8 : k + h * d.dim + (pl * 8 < d.dim ? pl * 8 : 0);
        krow[i] = c / NP;
        kld[i] = rot ? d.ldc : ldk;
    }
#pragma unroll
    for (int i = 0; i < VCH; i++) {
        const int c = t + T * i;
        voff[i] = min(c >> 3, d.vdim - 1) * ldv + (c & 7) * 8;
    }
    const bf16_t* vh = vt + (size_t)h * d.vdim * ldv;
    auto load = [&](int kb) {
#pragma unroll
        for (int i = 0; i < KCH; i++) rk[i] = *reinterpret_cast<const i32x4*>(kbase[i] + (size_t)(unsigned)(min(kb + krow[i], rows - 1) * kld[i]));
#pragma unroll
        for (int i = 0; i < VCH; i++) rv[i] = *reinterpret_cast<const i32x4*>(vh + kb + voff[i]);
    };
    load(kb0);
    for (int kb = kb0; kb <= kb1; kb += kFlashK) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < KCH; i++) {
            const int c = t + T * i;
            *reinterpret_cast<i32x4*>(lk + (c % NP) * KP + krow[i] * 16) = rk[i];
        }
#pragma unroll
        for (int i = 0; i < VCH; i++) {
            const int c = t + T * i;
            *reinterpret_cast<int2*>(lv + ((c & 7) * 2) * VP + (c >> 3) * 8) = make_int2(rv[i][0], rv[i][1]);
            *reinterpret_cast<int2*>(lv + ((c & 7) * 2 + 1) * VP + (c >> 3) * 8) = make_int2(rv[i][2], rv[i][3]);
        }
        __syncthreads();
        if (kb + kFlashK <= kb1) load(kb + kFlashK);
        const int kp = kv0 + kb;                          // position of the tile's first key
        if (kp > qmax || (d.window > 0 && kp + kFlashK - 1 < qmin - d.window + 1)) continue;
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
        if (kp + kFlashK - 1 > qmin || (d.window > 0 && kp < qmax - d.window + 1)) {     // the tile holds unseen keys
            const int far = d.window > 0 ? d.window : 0x7fffffff;
#pragma unroll
            for (int j = 0; j < 2; j++)
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    const int back = qp - (kp + j * 32 + (r >> 2) * 8 + half * 4 + (r & 3));
                    s[j][r] = (unsigned)back < (unsigned)far ? s[j][r] * sc2 : -INFINITY;
                    mx = fmaxf(mx, s[j][r]);
                }
        } else {
#pragma unroll
            for (int j = 0; j < 2; j++)
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    s[j][r] *= sc2;
                    mx = fmaxf(mx, s[j][r]);
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
                    const int8_t* src = lv + (j * 8 + st * 4 + half) * VP + (i * 32 + ln) * 8;
                    const uint2 a = *reinterpret_cast<const uint2*>(src), b = *reinterpret_cast<const uint2*>(src + 2 * VP);
                    const uint4 u = make_uint4(a.x, a.y, b.x, b.y);
                    const bf16x8 fv = *reinterpret_cast<const bf16x8*>(&u);
                    acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fv, ph, acc[i], 0, 0, 0);
                    acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fv, pl, acc[i], 0, 0, 0);
                }
            }
    }
    l += lane_xor_f<32>(l);
    const float inv = 1.0f / l;
    if (wq0 + ln < tokens) {
        bf16_t* dst = o + (size_t)(wq0 + ln) * ldo + h * d.vdim;
#pragma unroll
        for (int i = 0; i < NVT; i++)
#pragma unroll
            for (int g = 0; g < 4; g++) {
                const int v = i * 32 + g * 8 + half * 4;
                if (v < d.vdim) {
                    bf16x4 b;
#pragma unroll
                    for (int e = 0; e < 4; e++) b[e] = (bf16_t)(acc[i][g * 4 + e] * inv);
                    *reinterpret_cast<bf16x4*>(dst + v) = b;
                }
            }
    }
}

static int flash_dk(const LatentDims& d) { return (d.dim + 15) / 16 * 16 + (d.rot_dim + 15) / 16 * 16; }
bool latent_flash_ok(const LatentDims& d) {
    return d.dim % 8 == 0 && d.rot_dim % 8 == 0 && d.vdim % 4 == 0 && flash_dk(d) <= 256 && d.vdim <= 256;
}
int latent_flash(const LatentDims& d, const bf16_t* q, int ldq, const bf16_t* k, int ldk, const bf16_t* vt, int ldv, const bf16_t* cache,
                 int kv0, int pos0, int tokens, bf16_t* o, int ldo, hipStream_t st) {
    const int rows = pos0 + tokens - kv0;
    FX_REQUIRE(q && k && vt && cache && o && tokens > 0 && latent_flash_ok(d), "latent_flash: dim=%d rot=%d vdim=%d", d.dim, d.rot_dim, d.vdim);
    FX_REQUIRE((size_t)rows * ldk < (1ull << 31) && (size_t)rows * d.ldc < (1ull << 31) && (size_t)d.vdim * ldv < (1ull << 31), "latent_flash: %d rows", rows);
    FX_REQUIRE(ldq % 8 == 0 && ldk % 8 == 0 && ldv % 64 == 0 && ldv >= rows && ldo % 4 == 0 && kv0 >= 0 && pos0 >= kv0 && pos0 + tokens <= d.capacity,
               "latent_flash: strides %d %d %d %d, rows %d", ldq, ldk, ldv, ldo, rows);
    const int dk = flash_dk(d), dv = d.vdim, g4 = (tokens + 127) / 128 * d.heads, g2 = (tokens + 63) / 64 * d.heads;
    // two waves per workgroup where four would leave CUs without one
#define FX_FLASH(DK, DV)                                                                                                                   \
    do {                                                                                                                                   \
        if (g4 >= 256) latent_flash_kernel<DK, DV, 4><<<g4, 256, 0, st>>>(d, q, ldq, k, ldk, vt, ldv, cache, kv0, pos0, tokens, rows, o, ldo); \
        else latent_flash_kernel<DK, DV, 2><<<g2, 128, 0, st>>>(d, q, ldq, k, ldk, vt, ldv, cache, kv0, pos0, tokens, rows, o, ldo);         \
    } while (0)
    if (dk <= 64 && dv <= 64) FX_FLASH(64, 64);
    else if (dk <= 128 && dv <= 64) FX_FLASH(128, 64);
    else if (dk <= 128 && dv <= 128) FX_FLASH(128, 128);
    else if (dk <= 192 && dv <= 128) FX_FLASH(192, 128);
    else if (dv <= 128) FX_FLASH(256, 128);
    else FX_FLASH(256, 256);
#undef FX_FLASH
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

}  // namespace fx
