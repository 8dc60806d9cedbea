// Gated linear attention with a decay per key channel: S_t = diag(a_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, followed by
// the per-head RMS norm and the silu gate.  The state is float32 and lives in HBM between steps.
//
// One token at a time (any size): a workgroup per head walks the tokens.
// In chunks of C tokens, with L_t the running sum of log a inside a chunk (L <= 0 and falling):
//   state:  S_end = diag(e^{L_end}) S_0 + sum_t (k_t e^{L_end - L_t}) v_t^T
//   output: o_t = (q_t e^{L_t})^T S_0 + sum_{j<=t} A_tj v_j,  A_tj = sum_d q_td k_jd e^{L_td - L_jd}
// Every exponent that is formed is <= 0: A is cut into 16x16 blocks, a block left of the diagonal takes the running sum at
// its first row as common reference, a block on the diagonal forms the differences themselves.  Products run on
// v_mfma_f32_*_f32, so no operand is rounded.  Three kernels: the chunks' own contributions, the walk over chunks, the outputs.
#include "float_ops.h"

namespace fx {

// log of the decay of channel n (of heads x dim) from a token's low-rank gate input
template <typename ET>
__device__ __forceinline__ float gla_log_decay(const ET* __restrict__ w_a2, int ldw, const float* b, const float* a1, int n, int rank, float tau) {
    constexpr int CE = Chunk<ET>::N;
    float z = b[n];
    for (int r = 0; r < rank; r += CE) {
        float wv[CE];
        Chunk<ET>::unpack(*reinterpret_cast<const uint4*>(w_a2 + (size_t)n * ldw + r), wv);
#pragma unroll
        for (int e = 0; e < CE; e++)
            if (r + e < rank) z = fma_f(wv[e], a1[r + e], z);
    }
    return log_sigmoid_f(z) / tau;
}

// ---- one token after the other ---------------------------------------------------------------------------------------
constexpr int kGlaStepT = 512;
template <typename ET, typename PT, typename OT>
__global__ __launch_bounds__(kGlaStepT) void gla_step_kernel(GlaDims d, const PT* __restrict__ p, int ldp, const float* __restrict__ a1, int ld_a1,
                                                             const ET* __restrict__ w_a2, const float* __restrict__ b_a2,
                                                             const float* __restrict__ norm_w, float* __restrict__ state,
                                                             const int* __restrict__ pos_state, int tok0, int tokens, OT* __restrict__ o, int ldo) {
    extern __shared__ float sm[];                         // q, k, decay [dim]; sums [groups][vdim]; gate input [rank]
    __shared__ float red[kGlaStepT / 64];
    const int t = threadIdx.x, h = blockIdx.x, HD = d.heads * d.dim, HV = d.heads * d.vdim;
    float *sq = sm, *sk = sq + d.dim, *sa = sk + d.dim, *s1 = sa + d.dim, *sum = s1 + d.a_rank;
    const int cols = min(d.vdim, kGlaStepT), groups = kGlaStepT / cols, c0 = t % cols, g = t / cols;
    float* S = state + (size_t)h * d.dim * d.vdim;
    const float qs = 1.0f / sqrtf((float)d.dim);
    const int lda2 = pad_k(d.a_rank);
    for (int n = 0; n < tokens; n++) {
        const int tok = tok0 + n;
        const bool fresh = pos_state[0] + tok == 0;       // a sequence starts from a zero state
        const PT* row = p + (size_t)tok * ldp;
        __syncthreads();
        for (int i = t; i < d.a_rank; i += kGlaStepT) s1[i] = a1[(size_t)tok * ld_a1 + i];
        __syncthreads();
        for (int i = t; i < d.dim; i += kGlaStepT) {
            sq[i] = (float)row[h * d.dim + i] * qs;
            sk[i] = (float)row[HD + h * d.dim + i];
            sa[i] = exp_f<false>(gla_log_decay<ET>(w_a2, lda2, b_a2, s1, h * d.dim + i, d.a_rank, d.tau));
        }
        __syncthreads();
        for (int cb = 0; cb < d.vdim; cb += cols) {
            const int c = cb + c0;
            float acc = 0.0f;
            if (g < groups && c < d.vdim) {
                const float v = (float)row[2 * HD + h * d.vdim + c];
#pragma unroll 8
                for (int i = g; i < d.dim; i += groups) {
                    float s = fresh ? 0.0f : S[(size_t)i * d.vdim + c] * sa[i];
                    s = fma_f(sk[i], v, s);
                    S[(size_t)i * d.vdim + c] = s;
                    acc = fma_f(s, sq[i], acc);
                }
                sum[g * d.vdim + c] = acc;
            }
        }
        __syncthreads();
        float ss = 0.0f;
        for (int c = t; c < d.vdim; c += kGlaStepT) {
            float v = 0.0f;
            for (int i = 0; i < groups; i++) v += sum[i * d.vdim + c];
            sum[c] = v;                                   // only this thread reads column c of group 0
            ss = fma_f(v, v, ss);
        }
        const float rs = 1.0f / sqrtf(block_sum<kGlaStepT / 64>(ss, red) / (float)d.vdim + d.eps);
        for (int c = t; c < d.vdim; c += kGlaStepT) {
            const float gate = (float)row[2 * HD + HV + h * d.vdim + c];
            o[(size_t)tok * ldo + h * d.vdim + c] = (OT)(sum[c] * rs * norm_w[c] * (gate * sigmoid_f(gate)));
        }
    }
}

template <typename ET>
int gla_steps(const GlaDims& d, const void* p, int ldp, int p_f32, const float* a1, int ld_a1, const ET* w_a2, const float* b_a2,
              const float* norm_w, float* state, const int* pos_state, int tok0, int tokens, void* o, int ldo, int o_f32, hipStream_t st) {
    FX_REQUIRE(p && a1 && w_a2 && b_a2 && norm_w && state && pos_state && o && tokens > 0, "gla_steps: null pointer");
    const int cols = d.vdim < kGlaStepT ? d.vdim : kGlaStepT;
    const size_t lds = sizeof(float) * (3 * d.dim + d.a_rank + (size_t)(kGlaStepT / cols) * d.vdim);
    FX_REQUIRE(lds <= 60 * 1024, "gla_steps: dim=%d vdim=%d exceed LDS", d.dim, d.vdim);
#define FX_GLA(PT, OT) gla_step_kernel<ET, PT, OT><<<d.heads, kGlaStepT, lds, st>>>(d, static_cast<const PT*>(p), ldp, a1, ld_a1, w_a2, b_a2, norm_w, state, pos_state, tok0, tokens, static_cast<OT*>(o), ldo)
    if (p_f32 && o_f32) FX_GLA(float, float);
    else if (!p_f32 && !o_f32) FX_GLA(ET, ET);
    else { set_error("gla_steps: input and output are both float32 or both of the element type"); return FLEXLLM_EINVAL; }
#undef FX_GLA
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int gla_steps<bf16_t>(const GlaDims&, const void*, int, int, const float*, int, const bf16_t*, const float*, const float*, float*, const int*, int, int, void*, int, int, hipStream_t);
template int gla_steps<float>(const GlaDims&, const void*, int, int, const float*, int, const float*, const float*, const float*, float*, const int*, int, int, void*, int, int, hipStream_t);

// ---- chunks -----------------------------------------------------------------------------------------------------------
static __host__ __device__ constexpr int pad32(int v) { return (v + 31) / 32 * 32; }
bool gla_chunks_ok(const GlaDims& d) { return d.dim <= 256 && d.vdim <= 256 && d.a_rank <= 256; }
static int gla_chunk(const GlaDims& d) { return d.dim <= 128 && d.vdim <= 128 ? 64 : 32; }
size_t gla_chunk_scratch(const GlaDims& d, int tokens) {
    const size_t nc = (tokens + gla_chunk(d) - 1) / gla_chunk(d);
    return nc * d.heads * d.dim * ((size_t)d.vdim + 1);
}

// Running sums of log decay of one chunk and head into L [C][pitch]; rows beyond the chunk's n repeat the last one
// (their decay is 1), channels beyond dim are 0.
template <typename ET, int C>
__device__ __forceinline__ void gla_running_log(const GlaDims& d, const float* __restrict__ a1, int ld_a1, const ET* __restrict__ w_a2,
                                                const float* __restrict__ b_a2, int h, int tok0, int n, float* L, int pitch) {
    const int t = threadIdx.x, dp = pad32(d.dim), lda2 = pad_k(d.a_rank);
    for (int i = t; i < C * dp; i += 256) {
        const int r = i / dp, c = i - r * dp;
        L[r * pitch + c] = r < n && c < d.dim ? gla_log_decay<ET>(w_a2, lda2, b_a2, a1 + (size_t)(tok0 + r) * ld_a1, h * d.dim + c, d.a_rank, d.tau) : 0.0f;
    }
    __syncthreads();
    for (int c = t; c < dp; c += 256) {
        float s = 0.0f;
        for (int r = 0; r < C; r++) { s += L[r * pitch + c]; L[r * pitch + c] = s; }
    }
    __syncthreads();
}

// Contribution of a chunk to the state behind it, U [dim][vdim], and the chunk's whole decay.
template <typename ET, int C>
__global__ __launch_bounds__(256) void gla_chunk_state_kernel(GlaDims d, const ET* __restrict__ p, int ldp, const float* __restrict__ a1, int ld_a1,
                                                              const ET* __restrict__ w_a2, const float* __restrict__ b_a2, int tokens,
                                                              float* __restrict__ u_out, float* __restrict__ dec_out) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, ln = lane & 31, half = lane >> 5;
    const int h = blockIdx.x % d.heads, chunk = blockIdx.x / d.heads, tok0 = chunk * C, n = min(C, tokens - tok0);
    const int dp = pad32(d.dim), vp = pad32(d.vdim), HD = d.heads * d.dim;
    float *L = sm, *V = sm + C * dp;                      // L becomes the decayed keys
    gla_running_log<ET, C>(d, a1, ld_a1, w_a2, b_a2, h, tok0, n, L, dp);
    float* dec = dec_out + ((size_t)chunk * d.heads + h) * d.dim;
    for (int i = t; i < d.dim; i += 256) dec[i] = exp_f<false>(L[(C - 1) * dp + i]);
    for (int i = t; i < C * vp; i += 256) {
        const int r = i / vp, c = i - r * vp;
        V[i] = r < n && c < d.vdim ? (float)p[(size_t)(tok0 + r) * ldp + 2 * HD + h * d.vdim + c] : 0.0f;
    }
    __syncthreads();
    for (int c = t; c < dp; c += 256) {                   // column by column: the last row is needed until the end
        const float end = L[(C - 1) * dp + c];
        for (int r = 0; r < C; r++)
            L[r * dp + c] = r < n && c < d.dim ? (float)p[(size_t)(tok0 + r) * ldp + HD + h * d.dim + c] * exp_f<false>(end - L[r * dp + c]) : 0.0f;
    }
    __syncthreads();
    float* u = u_out + ((size_t)chunk * d.heads + h) * d.dim * d.vdim;
    const int nd = dp / 32, nv = vp / 32;
    for (int tile = wave; tile < nd * nv; tile += 4) {
        const int di = tile / nv * 32, vi = tile % nv * 32;
        f32x16 acc;
#pragma unroll
        for (int r = 0; r < 16; r++) acc[r] = 0.0f;
#pragma unroll 8
        for (int s = 0; s < C / 2; s++)
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(L[(2 * s + half) * dp + di + ln], V[(2 * s + half) * vp + vi + ln], acc, 0, 0, 0);
        const int col = vi + ln;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int row = di + (r >> 2) * 8 + half * 4 + (r & 3);
            if (row < d.dim && col < d.vdim) u[(size_t)row * d.vdim + col] = acc[r];
        }
    }
}

// Walk over the chunks: u[chunk] becomes the state in front of the chunk, `state` the one behind the last.
static __global__ __launch_bounds__(256) void gla_walk_kernel(int heads, int dim, int vdim, int chunks, float* __restrict__ u, const float* __restrict__ dec,
                                                              float* __restrict__ state, const int* __restrict__ pos_state) {
    const size_t per = (size_t)heads * dim * vdim, i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= per) return;
    const size_t hd = i / vdim;
    float s = pos_state[0] == 0 ? 0.0f : state[i];
    constexpr int B = 8;
    for (int c0 = 0; c0 < chunks; c0 += B) {
        float x[B], a[B];
#pragma unroll
        for (int b = 0; b < B; b++) {
            const int c = min(c0 + b, chunks - 1);
            x[b] = u[(size_t)c * per + i];
            a[b] = dec[(size_t)c * heads * dim + hd];
        }
#pragma unroll
        for (int b = 0; b < B; b++)
            if (c0 + b < chunks) {
                u[(size_t)(c0 + b) * per + i] = s;
                s = fma_f(a[b], s, x[b]);
            }
    }
    state[i] = s;
}

// Outputs of a chunk, with the head norm and the gate.
template <typename ET, int C>
__global__ __launch_bounds__(256) void gla_chunk_out_kernel(GlaDims d, const ET* __restrict__ p, int ldp, const float* __restrict__ a1, int ld_a1,
                                                            const ET* __restrict__ w_a2, const float* __restrict__ b_a2,
                                                            const float* __restrict__ norm_w, const float* __restrict__ u_in, int tokens,
                                                            ET* __restrict__ o, int ldo) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, ln = lane & 31, half = lane >> 5;
    const int h = blockIdx.x % d.heads, chunk = blockIdx.x / d.heads, tok0 = chunk * C, n = min(C, tokens - tok0);
    const int dp = pad32(d.dim), vp = pad32(d.vdim), P = dp + 1, VP = vp + 1, HD = d.heads * d.dim, HV = d.heads * d.vdim;
    constexpr int AP = C + 1;
    float *L = sm, *Q = L + C * P, *K = Q + C * P, *A = K + C * P;       // the outputs later take the room of L and Q
    gla_running_log<ET, C>(d, a1, ld_a1, w_a2, b_a2, h, tok0, n, L, P);
    const float qs = 1.0f / sqrtf((float)d.dim);
    for (int i = t; i < C * dp; i += 256) {
        const int r = i / dp, c = i - r * dp;
        const bool in = r < n && c < d.dim;
        const ET* row = p + (size_t)(tok0 + min(r, n - 1)) * ldp + h * d.dim;
        Q[r * P + c] = in ? (float)row[c] * qs : 0.0f;
        K[r * P + c] = in ? (float)row[HD + c] : 0.0f;
    }
    for (int i = t; i < C * AP; i += 256) A[i] = 0.0f;
    __syncthreads();
    // blocks of A on the diagonal: one (row, column) pair per thread
    constexpr int NB = C / 16;
    for (int i = t; i < NB * 256; i += 256) {
        const int b = i >> 8, r = b * 16 + ((i >> 4) & 15), c = b * 16 + (i & 15);
        if (c <= r) {
            float s = 0.0f;
            for (int e = 0; e < d.dim; e++) s = fma_f(Q[r * P + e] * K[c * P + e], exp_f<false>(L[r * P + e] - L[c * P + e]), s);
            A[r * AP + c] = s;
        }
    }
    // blocks left of it: 16x16 tiles on the matrix cores, operands scaled on the way in
    {
        constexpr int NT = NB * (NB - 1) / 2;
        for (int tile = wave; tile < NT; tile += 4) {
            int bi = 1, bj = tile;
            while (bj >= bi) { bj -= bi; bi++; }
            const int r = bi * 16 + (lane & 15), c = bj * 16 + (lane & 15), q4 = lane >> 4, ref = bi * 16 - 1;
            f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
            for (int e0 = 0; e0 < dp; e0 += 4) {
                const int e = e0 + q4;
                const float lr = L[ref * P + e];
                const float fa = Q[r * P + e] * exp_f<false>(L[r * P + e] - lr), fb = K[c * P + e] * exp_f<false>(lr - L[c * P + e]);
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(fa, fb, acc, 0, 0, 0);
            }
#pragma unroll
            for (int i = 0; i < 4; i++) A[(bi * 16 + q4 * 4 + i) * AP + c] = acc[i];
        }
    }
    __syncthreads();
    for (int i = t; i < C * dp; i += 256) {               // q_t e^{L_t} for the product with the state in front of the chunk
        const int r = i / dp, c = i - r * dp;
        Q[r * P + c] *= exp_f<false>(L[r * P + c]);
    }
    __syncthreads();
    const float* S = u_in + ((size_t)chunk * d.heads + h) * d.dim * d.vdim;
    const int nv = vp / 32;
    constexpr int NR = C / 32, kMaxMine = 2;              // at most 8 tiles: vdim <= 128 with two row tiles, <= 256 with one
    f32x16 acc[kMaxMine];
#pragma unroll
    for (int m = 0; m < kMaxMine; m++) {
        const int tile = wave + 4 * m;
#pragma unroll
        for (int r = 0; r < 16; r++) acc[m][r] = 0.0f;
        if (tile < NR * nv) {
            const int ri = tile / nv * 32, col = tile % nv * 32 + ln, cc = min(col, d.vdim - 1);
            const float cm = col < d.vdim ? 1.0f : 0.0f;
            for (int s = 0; s < dp / 2; s++) {
                const int e = 2 * s + half;
                acc[m] = __builtin_amdgcn_mfma_f32_32x32x2f32(Q[(ri + ln) * P + e], S[(size_t)min(e, d.dim - 1) * d.vdim + cc] * cm, acc[m], 0, 0, 0);
            }
            for (int s = 0; s < C / 2; s++) {
                const int j = 2 * s + half;
                const float v = j < n ? (float)p[(size_t)(tok0 + j) * ldp + 2 * HD + h * d.vdim + cc] * cm : 0.0f;
                acc[m] = __builtin_amdgcn_mfma_f32_32x32x2f32(A[(ri + ln) * AP + j], v, acc[m], 0, 0, 0);
            }
        }
    }
    __syncthreads();
    float* O = sm;                                        // [C][VP]
#pragma unroll
    for (int m = 0; m < kMaxMine; m++) {
        const int tile = wave + 4 * m;
        const int ri = tile / nv * 32, col = tile % nv * 32 + ln;
        if (tile < NR * nv)
#pragma unroll
        for (int r = 0; r < 16; r++) O[(ri + (r >> 2) * 8 + half * 4 + (r & 3)) * VP + col] = acc[m][r];
    }
    __syncthreads();
    for (int r = wave; r < n; r += 4) {
        float ss = 0.0f;
        for (int c = lane; c < d.vdim; c += 64) ss = fma_f(O[r * VP + c], O[r * VP + c], ss);
        const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)d.vdim + d.eps);
        for (int c = lane; c < d.vdim; c += 64) {
            const float gate = (float)p[(size_t)(tok0 + r) * ldp + 2 * HD + HV + h * d.vdim + c];
            o[(size_t)(tok0 + r) * ldo + h * d.vdim + c] = (ET)(O[r * VP + c] * rs * norm_w[c] * (gate * sigmoid_f(gate)));
        }
    }
}

template <typename ET, int C>
static int gla_chunks_c(const GlaDims& d, const ET* p, int ldp, const float* a1, int ld_a1, const ET* w_a2, const float* b_a2, const float* norm_w,
                        float* state, const int* pos_state, int tokens, float* scratch, ET* o, int ldo, hipStream_t st) {
    const int nc = (tokens + C - 1) / C, dp = pad32(d.dim), vp = pad32(d.vdim);
    float* u = scratch;
    float* dec = scratch + (size_t)nc * d.heads * d.dim * d.vdim;
    const size_t lds1 = sizeof(float) * C * (dp + vp);
    size_t lds3 = sizeof(float) * (3 * C * (dp + 1) + C * (C + 1));
    const size_t lds_o = sizeof(float) * C * (vp + 1);
    if (lds_o > lds3) lds3 = lds_o;
    FX_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(gla_chunk_state_kernel<ET, C>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1));
    FX_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(gla_chunk_out_kernel<ET, C>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds3));
    gla_chunk_state_kernel<ET, C><<<nc * d.heads, 256, lds1, st>>>(d, p, ldp, a1, ld_a1, w_a2, b_a2, tokens, u, dec);
    gla_walk_kernel<<<(int)(((size_t)d.heads * d.dim * d.vdim + 255) / 256), 256, 0, st>>>(d.heads, d.dim, d.vdim, nc, u, dec, state, pos_state);
    gla_chunk_out_kernel<ET, C><<<nc * d.heads, 256, lds3, st>>>(d, p, ldp, a1, ld_a1, w_a2, b_a2, norm_w, u, tokens, o, ldo);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template <typename ET>
int gla_chunks(const GlaDims& d, const ET* p, int ldp, const float* a1, int ld_a1, const ET* w_a2, const float* b_a2, const float* norm_w,
               float* state, const int* pos_state, int tokens, float* scratch, ET* o, int ldo, hipStream_t st) {
    FX_REQUIRE(p && a1 && w_a2 && b_a2 && norm_w && state && pos_state && scratch && o && tokens > 0, "gla_chunks: null pointer");
    FX_REQUIRE(gla_chunks_ok(d), "gla_chunks: dim=%d vdim=%d rank=%d (at most 256)", d.dim, d.vdim, d.a_rank);
    if (gla_chunk(d) == 64) return gla_chunks_c<ET, 64>(d, p, ldp, a1, ld_a1, w_a2, b_a2, norm_w, state, pos_state, tokens, scratch, o, ldo, st);
    return gla_chunks_c<ET, 32>(d, p, ldp, a1, ld_a1, w_a2, b_a2, norm_w, state, pos_state, tokens, scratch, o, ldo, st);
}
template int gla_chunks<bf16_t>(const GlaDims&, const bf16_t*, int, const float*, int, const bf16_t*, const float*, const float*, float*, const int*, int, float*, bf16_t*, int, hipStream_t);
template int gla_chunks<float>(const GlaDims&, const float*, int, const float*, int, const float*, const float*, const float*, float*, const int*, int, float*, float*, int, hipStream_t);

}  // namespace fx
