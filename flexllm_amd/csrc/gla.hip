// Gated linear attention with a decay per key channel: S_t = diag(a_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, followed by
// the per-head RMS norm and the silu gate.  The state is float32 and lives in HBM between steps.
//
// One token at a time (any size): a workgroup per head walks the tokens.
// In chunks of C tokens, with L_t the running sum of log a inside a chunk (L <= 0 and falling):
//   state:  S_end = diag(e^{L_end}) S_0 + sum_t (k_t e^{L_end - L_t}) v_t^T
//   output: o_t = (q_t e^{L_t})^T S_0 + sum_{j<=t} A_tj v_j,  A_tj = sum_d q_td k_jd e^{L_td - L_jd}
// Products run on v_mfma_f32_*_f32, so no operand is rounded.  Where a chunk's decay stays above e^-40 in every channel, A
// is the product of q e^{L} and k e^{-L}; otherwise A is cut into 16x16 blocks so that every exponent that is formed is
// <= 0: a block left of the diagonal takes the running sum at its first row as common reference, a block on the diagonal
// forms the differences themselves.  Kernels: running sums, the chunks' own contributions, the walk over chunks, the outputs.
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

// The same with the head's state in registers: 1024 threads, thread (g, c) holds a run of rows of column c.
// Everything that does not depend on the token's decay is requested at the start, in one trip to memory.
constexpr int kGlaRegT = 1024, kGlaRegRows = 16, kGlaRegRank = 16;
static bool gla_regs_ok(const GlaDims& d) {
    return d.vdim <= 512 && d.dim <= kGlaRegT && d.dim <= kGlaRegT / d.vdim * kGlaRegRows && d.a_rank <= 1024;
}
static __host__ __device__ int gla_reg_rows(int dim, int groups) { return ((dim + groups - 1) / groups + 3) / 4 * 4; }   // <= kGlaRegRows
template <typename ET, typename PT, typename OT>
__global__ __launch_bounds__(kGlaRegT) void gla_step_regs_kernel(GlaDims d, const PT* __restrict__ p, int ldp, const float* __restrict__ a1, int ld_a1,
                                                                 const ET* __restrict__ w_a2, const float* __restrict__ b_a2,
                                                                 const float* __restrict__ norm_w, float* __restrict__ state,
                                                                 const int* __restrict__ pos_state, int tok0, int tokens, OT* __restrict__ o, int ldo) {
    constexpr int CE = Chunk<ET>::N, NW = kGlaRegRank / CE;
    extern __shared__ __attribute__((aligned(16))) float sm[];     // q, k, decay [dim, padded]; gate input [rank]; sums [groups][vdim]
    __shared__ float red[kGlaRegT / 64];
    const int t = threadIdx.x, h = blockIdx.x, HD = d.heads * d.dim, HV = d.heads * d.vdim, lda2 = pad_k(d.a_rank);
    const int groups = kGlaRegT / d.vdim, c = t % d.vdim, g = t / d.vdim, rows = gla_reg_rows(d.dim, groups), dp = groups * rows, i0 = g * rows;
    float *sq = sm, *sk = sq + dp, *sa = sk + dp, *s1 = sa + dp, *sum = s1 + d.a_rank;
    const bool mine = g < groups, row_t = t < d.dim, col_t = t < d.vdim;
    float* S = state + (size_t)h * d.dim * d.vdim;
    const int pos = pos_state[0] + tok0;
    float s[kGlaRegRows];
#pragma unroll
    for (int j = 0; j < kGlaRegRows; j++) s[j] = mine && j < rows && i0 + j < d.dim ? S[(size_t)(i0 + j) * d.vdim + c] : 0.0f;
    for (int i = d.dim + t; i < dp; i += kGlaRegT) { sq[i] = 0.0f; sk[i] = 0.0f; sa[i] = 0.0f; }
    uint4 w[NW];
    const int ch = h * d.dim + t;
#pragma unroll
    for (int i = 0; i < NW; i++) w[i] = row_t ? *reinterpret_cast<const uint4*>(w_a2 + (size_t)ch * lda2 + i * CE) : make_uint4(0, 0, 0, 0);
    const float bias = row_t ? b_a2[ch] : 0.0f, nw = col_t ? norm_w[t] : 0.0f;
    const float qs = 1.0f / sqrtf((float)d.dim), inv_tau = 1.0f / d.tau;
    for (int n = 0; n < tokens; n++) {
        const PT* row = p + (size_t)(tok0 + n) * ldp;
        const float q = row_t ? (float)row[ch] : 0.0f, k = row_t ? (float)row[HD + ch] : 0.0f;
        const float v = mine ? (float)row[2 * HD + h * d.vdim + c] : 0.0f;
        const float gate = col_t ? (float)row[2 * HD + HV + h * d.vdim + t] : 0.0f;
        for (int i = t; i < d.a_rank; i += kGlaRegT) s1[i] = a1[(size_t)(tok0 + n) * ld_a1 + i];
        __syncthreads();
        if (row_t) {
            float z = bias;
#pragma unroll
            for (int i = 0; i < NW; i++) {
                float wv[CE];
                Chunk<ET>::unpack(w[i], wv);
#pragma unroll
                for (int e = 0; e < CE; e++)
                    if (i * CE + e < d.a_rank) z = fma_f(wv[e], s1[i * CE + e], z);
            }
            for (int r = kGlaRegRank; r < d.a_rank; r++) z = fma_f((float)w_a2[(size_t)ch * lda2 + r], s1[r], z);
            sq[t] = q * qs;
            sk[t] = k;
            sa[t] = exp_f<false>(log_sigmoid_f(z) * inv_tau);
        }
        __syncthreads();
        const bool fresh = pos + n == 0;                  // a sequence starts from a zero state
        float acc = 0.0f;
        if (mine)
#pragma unroll
            for (int j = 0; j < kGlaRegRows; j += 4) {
                if (j >= rows) break;
                const f32x4 k4 = *reinterpret_cast<const f32x4*>(sk + i0 + j), a4 = *reinterpret_cast<const f32x4*>(sa + i0 + j),
                            q4 = *reinterpret_cast<const f32x4*>(sq + i0 + j);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    s[j + e] = fma_f(k4[e], v, fresh ? 0.0f : s[j + e] * a4[e]);
                    acc = fma_f(s[j + e], q4[e], acc);
                }
            }
        if (mine) sum[g * d.vdim + c] = acc;
        __syncthreads();
        float x = 0.0f;
        if (col_t)
            for (int i = 0; i < groups; i++) x += sum[i * d.vdim + t];
        const float rs = 1.0f / sqrtf(block_sum<kGlaRegT / 64>(x * x, red) / (float)d.vdim + d.eps);
        if (col_t) o[(size_t)(tok0 + n) * ldo + h * d.vdim + t] = (OT)(x * rs * nw * (gate * sigmoid_f(gate)));
    }
#pragma unroll
    for (int j = 0; j < kGlaRegRows; j++)
        if (mine && j < rows && i0 + j < d.dim) S[(size_t)(i0 + j) * d.vdim + c] = s[j];
}

template <typename ET>
int gla_steps(const GlaDims& d, const void* p, int ldp, int p_f32, const float* a1, int ld_a1, const ET* w_a2, const float* b_a2,
              const float* norm_w, float* state, const int* pos_state, int tok0, int tokens, void* o, int ldo, int o_f32, hipStream_t st) {
    FX_REQUIRE(p && a1 && w_a2 && b_a2 && norm_w && state && pos_state && o && tokens > 0, "gla_steps: null pointer");
    if (gla_regs_ok(d)) {
        const int groups = kGlaRegT / d.vdim;
        const size_t lds = sizeof(float) * (3 * (size_t)groups * gla_reg_rows(d.dim, groups) + d.a_rank + (size_t)groups * d.vdim);
#define FX_GLA(PT, OT) gla_step_regs_kernel<ET, PT, OT><<<d.heads, kGlaRegT, lds, st>>>(d, static_cast<const PT*>(p), ldp, a1, ld_a1, w_a2, b_a2, norm_w, state, pos_state, tok0, tokens, static_cast<OT*>(o), ldo)
        FX_REQUIRE((p_f32 != 0) == (o_f32 != 0), "gla_steps: input and output are both float32 or both of the element type");
        if (p_f32) FX_GLA(float, float);
        else FX_GLA(ET, ET);
#undef FX_GLA
        FX_LAUNCH_CHECK();
        return FLEXLLM_OK;
    }
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
    // states in front of the chunks, decays of the chunks, running sums, one flag per chunk and head
    const size_t nc = (tokens + gla_chunk(d) - 1) / gla_chunk(d);
    return nc * d.heads * d.dim * ((size_t)d.vdim + 1) + nc * gla_chunk(d) * d.heads * d.dim + nc * d.heads + 64;
}

constexpr float kGlaMild = -40.0f;                        // smallest running sum for which e^{-L} is formed

// Running sums of log decay inside each chunk, cum [tokens][heads * dim].  64 channels per workgroup; a wave takes a quarter
// of the chunk's tokens and adds the earlier quarters' totals at the end.
template <typename ET, int RMAX, int C>
__global__ __launch_bounds__(256) void gla_cum_kernel(GlaDims d, const float* __restrict__ a1, int ld_a1, const ET* __restrict__ w_a2,
                                                      const float* __restrict__ b_a2, int tokens, float* __restrict__ cum) {
    constexpr bool kRegs = RMAX > 0;
    constexpr int Q = C / 4;
    const int rp = kRegs ? RMAX : d.a_rank;               // row length in LDS, zero beyond the rank
    extern __shared__ __attribute__((aligned(16))) float s1[];
    __shared__ float total[4][64];
    const int t = threadIdx.x, tok0 = blockIdx.x * C, n = min(C, tokens - tok0), HD = d.heads * d.dim, ch = blockIdx.y * 64 + (t & 63), q = t >> 6;
    for (int i = t; i < n * rp; i += 256) {
        const int r = i / rp, c = i - r * rp;
        s1[i] = c < d.a_rank ? a1[(size_t)(tok0 + r) * ld_a1 + c] : 0.0f;
    }
    const ET* w = w_a2 + (size_t)min(ch, HD - 1) * pad_k(d.a_rank);
    const float b = b_a2[min(ch, HD - 1)], inv = 1.0f / d.tau;
    float wr[kRegs ? RMAX : 1];
    if constexpr (kRegs) {                                // the weights' rows are padded with zeros to 64 columns
        constexpr int CE = Chunk<ET>::N;
#pragma unroll
        for (int r = 0; r < RMAX; r += CE) {
            float v[CE];
            Chunk<ET>::unpack(*reinterpret_cast<const uint4*>(w + r), v);
#pragma unroll
            for (int e = 0; e < CE; e++) wr[r + e] = v[e];
        }
    }
    __syncthreads();
    float run[Q], s = 0.0f;
#pragma unroll
    for (int j = 0; j < Q; j++) {
        const int i = min(q * Q + j, n - 1);
        float z = b;
        if constexpr (kRegs) {
#pragma unroll
            for (int r = 0; r < RMAX; r += 4) {
                const f32x4 x = *reinterpret_cast<const f32x4*>(s1 + i * RMAX + r);
#pragma unroll
                for (int e = 0; e < 4; e++) z = fma_f(wr[r + e], x[e], z);
            }
        } else {
            for (int r = 0; r < d.a_rank; r++) z = fma_f((float)w[r], s1[i * d.a_rank + r], z);
        }
        s += log_sigmoid_f(z) * inv;
        run[j] = s;
    }
    total[q][t & 63] = s;
    __syncthreads();
    float before = 0.0f;
    for (int i = 0; i < q; i++) before += total[i][t & 63];
    if (ch >= HD) return;
#pragma unroll
    for (int j = 0; j < Q; j++)
        if (q * Q + j < n) cum[(size_t)(tok0 + q * Q + j) * HD + ch] = run[j] + before;
}

// Contribution of a chunk to the state behind it, U [dim][vdim], the chunk's whole decay, and whether the decay is mild.
// Any size.
template <typename ET, int C>
__global__ __launch_bounds__(256) void gla_chunk_state_kernel(GlaDims d, const ET* __restrict__ p, int ldp, const float* __restrict__ cum, int tokens,
                                                              float* __restrict__ u_out, float* __restrict__ dec_out, int* __restrict__ mild) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, ln = lane & 31, half = lane >> 5;
    const int h = blockIdx.x % d.heads, chunk = blockIdx.x / d.heads, tok0 = chunk * C, n = min(C, tokens - tok0);
    const int dp = pad32(d.dim), vp = pad32(d.vdim), HD = d.heads * d.dim;
    float *K = sm, *V = sm + C * dp;
    const float* L = cum + (size_t)tok0 * HD + h * d.dim;
    float* dec = dec_out + ((size_t)chunk * d.heads + h) * d.dim;
    int ok = 1;
    for (int i = t; i < d.dim; i += 256) {
        const float e = L[(size_t)(n - 1) * HD + i];
        dec[i] = exp_f<false>(e);
        ok &= e > kGlaMild;
    }
    ok = __syncthreads_and(ok);
    if (t == 0) mild[chunk * d.heads + h] = ok;
    for (int i = t; i < C * vp; i += 256) {
        const int r = i / vp, c = i - r * vp;
        V[i] = r < n && c < d.vdim ? (float)p[(size_t)(tok0 + r) * ldp + 2 * HD + h * d.vdim + c] : 0.0f;
    }
    for (int i = t; i < C * dp; i += 256) {
        const int r = i / dp, c = i - r * dp;
        K[i] = r < n && c < d.dim ? (float)p[(size_t)(tok0 + r) * ldp + HD + h * d.dim + c] * exp_f<false>(L[(size_t)(n - 1) * HD + c] - L[(size_t)r * HD + c]) : 0.0f;
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
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(K[(2 * s + half) * dp + di + ln], V[(2 * s + half) * vp + vi + ln], acc, 0, 0, 0);
        const int col = vi + ln;
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int row = di + (r >> 2) * 8 + half * 4 + (r & 3);
            if (row < d.dim && col < d.vdim) u[(size_t)row * d.vdim + col] = acc[r];
        }
    }
}

// One thread's 16-byte pieces of a [64][D] bfloat16 tile whose rows lie ld apart: piece i of thread t is row
// (t + 256 i) / (D / 8), columns 8 ((t + 256 i) % (D / 8)) ..; rows from n and columns from w on are zero.
template <int D>
struct GlaTile {
    static constexpr int PC = D / 8, NP = 64 * PC / 256;
    uint4 u[NP];
    __device__ __forceinline__ static int row(int i) { return ((int)threadIdx.x + 256 * i) / PC; }
    __device__ __forceinline__ static int col(int i) { return ((int)threadIdx.x + 256 * i) % PC * 8; }
    __device__ __forceinline__ void load(const bf16_t* base, int ld, int n, int w) {
#pragma unroll
        for (int i = 0; i < NP; i++)
            u[i] = row(i) < n && col(i) < w ? *reinterpret_cast<const uint4*>(base + (size_t)row(i) * ld + col(i)) : make_uint4(0, 0, 0, 0);
    }
};
template <int D>
struct GlaCum {                                           // the matching float32 running sums; rows from n on repeat row n-1
    f32x4 v[GlaTile<D>::NP][2];
    __device__ __forceinline__ void load(const float* base, int ld, int n, int w) {
#pragma unroll
        for (int i = 0; i < GlaTile<D>::NP; i++) {
            const float* p = base + (size_t)min(GlaTile<D>::row(i), n - 1) * ld + GlaTile<D>::col(i);
            const bool in = GlaTile<D>::col(i) < w;
            v[i][0] = in ? *reinterpret_cast<const f32x4*>(p) : f32x4{0, 0, 0, 0};
            v[i][1] = in ? *reinterpret_cast<const f32x4*>(p + 4) : f32x4{0, 0, 0, 0};
        }
    }
};

// The same as gla_chunk_state_kernel for bfloat16, dim and vdim multiples of 8 up to D: every load is 16 bytes and is in
// flight before the first is used.
template <int D>
__global__ __launch_bounds__(256) void gla_chunk_state_vec_kernel(GlaDims d, const bf16_t* __restrict__ p, int ldp, const float* __restrict__ cum, int tokens,
                                                                  float* __restrict__ u_out, float* __restrict__ dec_out, int* __restrict__ mild) {
    constexpr int C = 64, NT = D / 32;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, ln = lane & 31, half = lane >> 5;
    const int h = blockIdx.x % d.heads, chunk = blockIdx.x / d.heads, tok0 = chunk * C, n = min(C, tokens - tok0), HD = d.heads * d.dim;
    float *K = sm, *V = sm + C * D;
    const float* L = cum + (size_t)tok0 * HD + h * d.dim;
    const bf16_t* row = p + (size_t)tok0 * ldp;
    GlaTile<D> tk, tv;
    GlaCum<D> tl;
    tl.load(L, HD, n, d.dim);
    tk.load(row + HD + h * d.dim, ldp, n, d.dim);
    tv.load(row + 2 * HD + h * d.vdim, ldp, n, d.vdim);
    f32x4 end[2];                                         // D / 8 divides 256: the columns are the same in every piece
    {
        const float* e = L + (size_t)(n - 1) * HD + GlaTile<D>::col(0);
        const bool in = GlaTile<D>::col(0) < d.dim;
        end[0] = in ? *reinterpret_cast<const f32x4*>(e) : f32x4{0, 0, 0, 0};
        end[1] = in ? *reinterpret_cast<const f32x4*>(e + 4) : f32x4{0, 0, 0, 0};
    }
    int ok = 1;
#pragma unroll
    for (int e = 0; e < 8; e++) ok &= end[e >> 2][e & 3] > kGlaMild;
    if (t < GlaTile<D>::PC && GlaTile<D>::col(0) < d.dim) {
        float* dec = dec_out + ((size_t)chunk * d.heads + h) * d.dim + t * 8;
#pragma unroll
        for (int e = 0; e < 8; e++) dec[e] = exp_f<false>(end[e >> 2][e & 3]);
    }
    ok = __syncthreads_and(ok);
    if (t == 0) mild[chunk * d.heads + h] = ok;
#pragma unroll
    for (int i = 0; i < GlaTile<D>::NP; i++) {
        const int o = GlaTile<D>::row(i) * D + GlaTile<D>::col(i);
        float k[8], v[8];
        Chunk<bf16_t>::unpack(tk.u[i], k);
        Chunk<bf16_t>::unpack(tv.u[i], v);
#pragma unroll
        for (int g = 0; g < 2; g++) {
            f32x4 x, y;
#pragma unroll
            for (int e = 0; e < 4; e++) { x[e] = k[g * 4 + e] * exp_f<false>(end[g][e] - tl.v[i][g][e]); y[e] = v[g * 4 + e]; }
            *reinterpret_cast<f32x4*>(K + o + g * 4) = x;
            *reinterpret_cast<f32x4*>(V + o + g * 4) = y;
        }
    }
    __syncthreads();
    // a wave owns a column tile of the values and its channel tiles: the value operand is read once for all of them
    float* u = u_out + ((size_t)chunk * d.heads + h) * d.dim * d.vdim;
    constexpr int MT = NT * NT / 4;                       // tiles per wave: a column of four, or one of the four
    const int vt = wave % NT, i0 = wave / NT;             // (two column tiles: waves 2 and 3 take the second channel tile)
    f32x16 acc[MT];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) acc[i][r] = 0.0f;
#pragma unroll 4
    for (int s = 0; s < C / 2; s++) {
        const float b = V[(2 * s + half) * D + vt * 32 + ln];
#pragma unroll
        for (int i = 0; i < MT; i++) acc[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(K[(2 * s + half) * D + (i0 + i) * 32 + ln], b, acc[i], 0, 0, 0);
    }
    const int col = vt * 32 + ln;
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int rw = (i0 + i) * 32 + (r >> 2) * 8 + half * 4 + (r & 3);
            if (rw < d.dim && col < d.vdim) u[(size_t)rw * d.vdim + col] = acc[i][r];
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

// Outputs of a chunk, with the head norm and the gate.  Any size and any decay.  skip_mild: leave chunks with a mild
// decay to gla_chunk_out_vec_kernel.
template <typename ET, int C>
__global__ __launch_bounds__(256) void gla_chunk_out_kernel(GlaDims d, const ET* __restrict__ p, int ldp, const float* __restrict__ cum,
                                                            const float* __restrict__ norm_w, const float* __restrict__ u_in, int tokens,
                                                            ET* __restrict__ o, int ldo, const int* __restrict__ mild, int skip_mild) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, ln = lane & 31, half = lane >> 5;
    const int h = blockIdx.x % d.heads, chunk = blockIdx.x / d.heads, tok0 = chunk * C, n = min(C, tokens - tok0);
    if (skip_mild && mild[chunk * d.heads + h]) return;
    const int dp = pad32(d.dim), vp = pad32(d.vdim), P = dp + 1, VP = vp + 1, HD = d.heads * d.dim, HV = d.heads * d.vdim;
    constexpr int AP = C + 1;
    float *L = sm, *Q = L + C * P, *K = Q + C * P, *A = K + C * P;       // the outputs later take the room of L and Q
    const float qs = 1.0f / sqrtf((float)d.dim);
    for (int i = t; i < C * dp; i += 256) {
        const int r = i / dp, c = i - r * dp, rr = min(r, n - 1);
        const bool in = r < n && c < d.dim;
        const ET* row = p + (size_t)(tok0 + rr) * ldp + h * d.dim;
        Q[r * P + c] = in ? (float)row[c] * qs : 0.0f;
        K[r * P + c] = in ? (float)row[HD + c] : 0.0f;
        L[r * P + c] = c < d.dim ? cum[(size_t)(tok0 + rr) * HD + h * d.dim + c] : 0.0f;
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

// The same for bfloat16, a mild decay, dim and vdim multiples of 8 up to D (64 or 128).  q e^{L} serves both products; the
// room of k e^{-L} in LDS is taken over by A and the values once A stands in registers.
template <int D>
__global__ __launch_bounds__(256) void gla_chunk_out_vec_kernel(GlaDims d, const bf16_t* __restrict__ p, int ldp, const float* __restrict__ cum,
                                                                const float* __restrict__ norm_w, const float* __restrict__ u_in, int tokens,
                                                                bf16_t* __restrict__ o, int ldo, const int* __restrict__ mild) {
    constexpr int C = 64, P = D + 2, AP = C + 2, NT = D / 32;   // pitches = 2 modulo 64 banks: the 32x2 operand reads hit every bank once
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, ln = lane & 31, half = lane >> 5;
    const int h = blockIdx.x % d.heads, chunk = blockIdx.x / d.heads, tok0 = chunk * C, n = min(C, tokens - tok0);
    if (!mild[chunk * d.heads + h]) return;
    const int HD = d.heads * d.dim, HV = d.heads * d.vdim;
    float *Q = sm, *K = sm + C * P, *A = K;
    bf16_t* V = reinterpret_cast<bf16_t*>(K + C * AP);    // [64][D] behind A
    static_assert(C * AP + C * D / 2 <= (D == 64 ? 2 : 1) * C * P, "A and the values fit into the keys' room");
    const bf16_t* row = p + (size_t)tok0 * ldp;
    GlaTile<D> tq, tk, tv, tg;
    GlaCum<D> tl;
    tl.load(cum + (size_t)tok0 * HD + h * d.dim, HD, n, d.dim);
    tq.load(row + h * d.dim, ldp, n, d.dim);
    tk.load(row + HD + h * d.dim, ldp, n, d.dim);
    tv.load(row + 2 * HD + h * d.vdim, ldp, n, d.vdim);
    const float qs = 1.0f / sqrtf((float)d.dim);
#pragma unroll
    for (int i = 0; i < GlaTile<D>::NP; i++) {
        const int off = GlaTile<D>::row(i) * P + GlaTile<D>::col(i);
        float q[8], k[8];
        Chunk<bf16_t>::unpack(tq.u[i], q);
        Chunk<bf16_t>::unpack(tk.u[i], k);
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
            const float l0 = tl.v[i][e >> 2][e & 3], l1 = tl.v[i][e >> 2][(e & 3) + 1];
            *reinterpret_cast<float2*>(Q + off + e) = make_float2(q[e] * qs * exp_f<false>(l0), q[e + 1] * qs * exp_f<false>(l1));
            *reinterpret_cast<float2*>(K + off + e) = make_float2(k[e] * exp_f(-l0), k[e + 1] * exp_f(-l1));
        }
    }
    __syncthreads();
    // A: the ten 16x16 tiles on and below the diagonal, walked by the four waves
    f32x4 a[3];
#pragma unroll
    for (int m = 0; m < 3; m++) {
        const int tile = wave + 4 * m;
        a[m] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        if (tile < 10) {
            const int bi = tile < 1 ? 0 : tile < 3 ? 1 : tile < 6 ? 2 : 3, bj = tile - bi * (bi + 1) / 2;
            const int r = bi * 16 + (lane & 15), c = bj * 16 + (lane & 15), q4 = lane >> 4;
#pragma unroll 8
            for (int e = 0; e < D; e += 4) a[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(Q[r * P + e + q4], K[c * P + e + q4], a[m], 0, 0, 0);
        }
    }
    __syncthreads();
    for (int i = t; i < C * AP; i += 256) A[i] = 0.0f;
    __syncthreads();
#pragma unroll
    for (int m = 0; m < 3; m++) {
        const int tile = wave + 4 * m;
        if (tile < 10) {
            const int bi = tile < 1 ? 0 : tile < 3 ? 1 : tile < 6 ? 2 : 3, bj = tile - bi * (bi + 1) / 2, c = bj * 16 + (lane & 15);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int r = bi * 16 + (lane >> 4) * 4 + i;
                if (c <= r) A[r * AP + c] = a[m][i];
            }
        }
    }
#pragma unroll
    for (int i = 0; i < GlaTile<D>::NP; i++) {
        uint2* dst = reinterpret_cast<uint2*>(V + GlaTile<D>::row(i) * D + GlaTile<D>::col(i));
        dst[0] = make_uint2(tv.u[i].x, tv.u[i].y);
        dst[1] = make_uint2(tv.u[i].z, tv.u[i].w);
    }
    tg.load(row + 2 * HD + HV + h * d.vdim, ldp, n, d.vdim);    // the gates, in flight during the products
    __syncthreads();
    // a wave owns a column tile and both row tiles (D = 128), or one row tile (D = 64: two column tiles)
    constexpr int MR = NT >= 4 ? 2 : 1;
    const int vt = NT >= 4 ? wave : wave & 1, r0 = NT >= 4 ? 0 : (wave >> 1) * 32;
    f32x16 acc[MR];
#pragma unroll
    for (int i = 0; i < MR; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) acc[i][r] = 0.0f;
    const float* S = u_in + ((size_t)chunk * d.heads + h) * d.dim * d.vdim;
    const int col = vt * 32 + ln, cc = min(col, d.vdim - 1);
    constexpr int B = 16;                                 // state rows in flight per lane
    float sb[2][B];
    auto load_state = [&](int e0, float (&x)[B]) {
#pragma unroll
        for (int i = 0; i < B; i++) x[i] = S[(size_t)min(e0 + 2 * i + half, d.dim - 1) * d.vdim + cc];
    };
    load_state(0, sb[0]);
#pragma unroll
    for (int e0 = 0; e0 < D; e0 += 2 * B) {
        constexpr int STEPS = D / (2 * B);
        const int cur = (e0 / (2 * B)) & 1;
        if (e0 / (2 * B) + 1 < STEPS) load_state(e0 + 2 * B, sb[cur ^ 1]);
#pragma unroll
        for (int i = 0; i < B; i++)
#pragma unroll
            for (int m = 0; m < MR; m++)
                acc[m] = __builtin_amdgcn_mfma_f32_32x32x2f32(Q[(r0 + m * 32 + ln) * P + e0 + 2 * i + half], sb[cur][i], acc[m], 0, 0, 0);
    }
#pragma unroll 8
    for (int s = 0; s < C / 2; s++) {
        const int j = 2 * s + half;
        const float v = (float)V[j * D + vt * 32 + ln];
#pragma unroll
        for (int m = 0; m < MR; m++) acc[m] = __builtin_amdgcn_mfma_f32_32x32x2f32(A[(r0 + m * 32 + ln) * AP + j], v, acc[m], 0, 0, 0);
    }
    __syncthreads();
    float* O = Q;                                         // [64][P]
#pragma unroll
    for (int m = 0; m < MR; m++)
#pragma unroll
        for (int r = 0; r < 16; r++) O[(r0 + m * 32 + (r >> 2) * 8 + half * 4 + (r & 3)) * P + col] = col < d.vdim ? acc[m][r] : 0.0f;
    __syncthreads();
    // head norm: D / 8 neighbouring threads share a row
    constexpr int PC = D / 8;
#pragma unroll
    for (int i = 0; i < GlaTile<D>::NP; i++) {
        const int r = GlaTile<D>::row(i), c = GlaTile<D>::col(i);
        float x[8], g[8], ss = 0.0f;
#pragma unroll
        for (int e = 0; e < 8; e++) { x[e] = O[r * P + c + e]; ss = fma_f(x[e], x[e], ss); }
        ss += lane_xor_f<1>(ss);
        ss += lane_xor_f<2>(ss);
        ss += lane_xor_f<4>(ss);
        if constexpr (PC == 16) ss += lane_xor_f<8>(ss);
        const float rs = 1.0f / sqrtf(ss / (float)d.vdim + d.eps);
        if (r < n && c < d.vdim) {
            Chunk<bf16_t>::unpack(tg.u[i], g);
            bf16x8 out;
#pragma unroll
            for (int e = 0; e < 8; e++) out[e] = (bf16_t)(x[e] * rs * norm_w[c + e] * (g[e] * sigmoid_f(g[e])));
            *reinterpret_cast<bf16x8*>(o + (size_t)(tok0 + r) * ldo + h * d.vdim + c) = out;
        }
    }
}

template <typename F>
static int opt_in_lds(F* f, size_t bytes) {
    FX_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(f), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
    return FLEXLLM_OK;
}

template <typename ET, int C>
static int gla_chunks_c(const GlaDims& d, const ET* p, int ldp, const float* a1, int ld_a1, const ET* w_a2, const float* b_a2, const float* norm_w,
                        float* state, const int* pos_state, int tokens, float* scratch, ET* o, int ldo, hipStream_t st) {
    const int nc = (tokens + C - 1) / C, dp = pad32(d.dim), vp = pad32(d.vdim), HD = d.heads * d.dim;
    float* u = scratch;
    float* dec = u + (size_t)nc * HD * d.vdim;
    float* cum = dec + ((size_t)nc * HD + 15) / 16 * 16;
    int* mild = reinterpret_cast<int*>(cum + (size_t)nc * C * HD);
    int rc;
    {
        const dim3 grid(nc, (HD + 63) / 64);
        const size_t lds = sizeof(float) * C * (d.a_rank <= 16 ? 16 : d.a_rank <= 32 ? 32 : d.a_rank);
        if (d.a_rank <= 16) gla_cum_kernel<ET, 16, C><<<grid, 256, lds, st>>>(d, a1, ld_a1, w_a2, b_a2, tokens, cum);
        else if (d.a_rank <= 32) gla_cum_kernel<ET, 32, C><<<grid, 256, lds, st>>>(d, a1, ld_a1, w_a2, b_a2, tokens, cum);
        else gla_cum_kernel<ET, 0, C><<<grid, 256, lds, st>>>(d, a1, ld_a1, w_a2, b_a2, tokens, cum);
    }
    const int walk = (int)(((size_t)HD * d.vdim + 255) / 256);
    bool vec = false;
    if constexpr (std::is_same<ET, bf16_t>::value && C == 64) {
        vec = d.dim % 8 == 0 && d.vdim % 8 == 0 && ldp % 8 == 0 && ldo % 8 == 0;
        if (vec) {
            const bool wide = d.dim > 64 || d.vdim > 64;
            const size_t ls = sizeof(float) * 2 * C * (wide ? 128 : 64), lo = sizeof(float) * (wide ? 2 * C * 130 : 3 * C * 66);
            if (wide) {
                if ((rc = opt_in_lds(gla_chunk_state_vec_kernel<128>, ls)) || (rc = opt_in_lds(gla_chunk_out_vec_kernel<128>, lo))) return rc;
                gla_chunk_state_vec_kernel<128><<<nc * d.heads, 256, ls, st>>>(d, p, ldp, cum, tokens, u, dec, mild);
                gla_walk_kernel<<<walk, 256, 0, st>>>(d.heads, d.dim, d.vdim, nc, u, dec, state, pos_state);
                gla_chunk_out_vec_kernel<128><<<nc * d.heads, 256, lo, st>>>(d, p, ldp, cum, norm_w, u, tokens, o, ldo, mild);
            } else {
                if ((rc = opt_in_lds(gla_chunk_state_vec_kernel<64>, ls)) || (rc = opt_in_lds(gla_chunk_out_vec_kernel<64>, lo))) return rc;
                gla_chunk_state_vec_kernel<64><<<nc * d.heads, 256, ls, st>>>(d, p, ldp, cum, tokens, u, dec, mild);
                gla_walk_kernel<<<walk, 256, 0, st>>>(d.heads, d.dim, d.vdim, nc, u, dec, state, pos_state);
                gla_chunk_out_vec_kernel<64><<<nc * d.heads, 256, lo, st>>>(d, p, ldp, cum, norm_w, u, tokens, o, ldo, mild);
            }
        }
    }
    size_t lds3 = sizeof(float) * (3 * C * (dp + 1) + C * (C + 1));
    const size_t lds1 = sizeof(float) * C * (dp + vp), lds_o = sizeof(float) * C * (vp + 1);
    if (lds_o > lds3) lds3 = lds_o;
    if ((rc = opt_in_lds(gla_chunk_state_kernel<ET, C>, lds1)) || (rc = opt_in_lds(gla_chunk_out_kernel<ET, C>, lds3))) return rc;
    if (!vec) {
        gla_chunk_state_kernel<ET, C><<<nc * d.heads, 256, lds1, st>>>(d, p, ldp, cum, tokens, u, dec, mild);
        gla_walk_kernel<<<walk, 256, 0, st>>>(d.heads, d.dim, d.vdim, nc, u, dec, state, pos_state);
    }
    gla_chunk_out_kernel<ET, C><<<nc * d.heads, 256, lds3, st>>>(d, p, ldp, cum, norm_w, u, tokens, o, ldo, mild, vec ? 1 : 0);
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
