// Linears of one token: y = W h with W of ET (bfloat16 or float32) streamed once, h float32 in LDS.
//
// A workgroup of 256 threads owns R weight rows; thread t reads 16-byte pieces t, t + 256, ... of each.  The first
// R x S pieces are requested before the prologue (residual, norms, expert choice) runs, so that its latency lies under
// the weight stream.  The R sums are reduced together (multi_sum_step).
#include "float_ops.h"

namespace fx {

constexpr int kMaxExperts = 1024, kMaxTop = 32;

// Expert choice of one token by one wave: softmax over the router outputs, the `top` largest (ties: lower index), their
// weights divided by their sum.  sel / wt: LDS, filled by every lane's agreement (lane 0 writes).
__device__ __forceinline__ void route_wave(const float* __restrict__ z, int experts, int top, int* sel, float* wt) {
    const int lane = threadIdx.x & 63;
    float v[kMaxExperts / 64];
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < kMaxExperts / 64; i++) {
        const int e = i * 64 + lane;
        v[i] = -INFINITY;
        if (i * 64 < experts && e < experts) v[i] = z[e];
        mx = fmaxf(mx, v[i]);
    }
    mx = wave_max(mx);
    float den = 0.0f;
#pragma unroll
    for (int i = 0; i < kMaxExperts / 64; i++) {
        if (i * 64 >= experts) break;
        v[i] = i * 64 + lane < experts ? exp_f(v[i] - mx) : -1.0f;
        den += fmaxf(v[i], 0.0f);
    }
    den = wave_sum(den);
    float sum = 0.0f;
    for (int k = 0; k < top; k++) {
        float best = -2.0f;
        int bi = 0x7fffffff;
#pragma unroll
        for (int i = 0; i < kMaxExperts / 64; i++) {
            if (i * 64 >= experts) break;
            if (v[i] > best) { best = v[i]; bi = i * 64 + lane; }
        }
#pragma unroll
        for (int m = 1; m < 64; m <<= 1) {
            const float ov = __shfl_xor(best, m);
            const int oi = __shfl_xor(bi, m);
            if (ov > best || (ov == best && oi < bi)) { best = ov; bi = oi; }
        }
#pragma unroll
        for (int i = 0; i < kMaxExperts / 64; i++) {
            if (i * 64 >= experts) break;
            if (i * 64 + lane == bi) v[i] = -1.0f;
        }
        const float s = best / den;
        sum += s;
        if (lane == 0) { sel[k] = bi; wt[k] = s; }
    }
    if (lane == 0)
        for (int k = 0; k < top; k++) wt[k] = wt[k] / (sum + 1e-20f);
}

template <typename ET, int R, int S, int PRO>
__global__ __launch_bounds__(256) void gemv_float_kernel(GemvArgs g) {
    constexpr int CE = Chunk<ET>::N;
    extern __shared__ __attribute__((aligned(16))) float xs[];     // [kpad] the vector, then the reduction area
    __shared__ float red[4 * (R > 4 ? R : 4)];
    __shared__ int sel[kMaxTop];
    __shared__ float wt[kMaxTop];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int tok = PRO == 2 ? blockIdx.y / g.top : blockIdx.y;
    const int row0 = blockIdx.x * R;
    const ET* w = static_cast<const ET*>(g.w);
    if constexpr (PRO == 2) {
        if (wave == 0) route_wave(g.route + (size_t)tok * g.ld_route, g.experts, g.top, sel, wt);
        __syncthreads();
        const int slot = blockIdx.y % g.top;
        w += (size_t)__builtin_amdgcn_readfirstlane(sel[slot]) * g.w_stride;
        if (blockIdx.x == 0 && t == 0) { g.pick[blockIdx.y] = sel[slot]; g.pick_w[blockIdx.y] = wt[slot]; }
    }
    const int nchunk = g.kpad / CE;                       // 16-byte pieces of a row
    uint4 pre[R][S];
#pragma unroll
    for (int r = 0; r < R; r++)
#pragma unroll
        for (int s = 0; s < S; s++) {
            const int c = s * 256 + t;
            pre[r][s] = c < nchunk ? *reinterpret_cast<const uint4*>(w + (size_t)min(row0 + r, g.n - 1) * g.kpad + c * CE)
                                   : make_uint4(0, 0, 0, 0);
        }
    // ---- the vector
    const float* x = g.x + (size_t)tok * g.ldx;
    if constexpr (PRO == 1) {
        float rs = 0.0f;
        if (g.y) {
            const float* y = g.y + (size_t)tok * g.ldy;
            float ss = 0.0f;
            for (int i = t; i < g.k; i += 256) { const float v = y[i]; xs[i] = v; ss = fma_f(v, v, ss); }
            rs = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)g.k + g.eps);
        }
        float ss = 0.0f;
        for (int i = t; i < g.k; i += 256) {
            float v = x[i];
            if (g.y) v = v + xs[i] * rs * g.gb[i];
            xs[i] = v;
            ss = fma_f(v, v, ss);
            if (blockIdx.x == 0 && g.x_new) g.x_new[(size_t)tok * g.ldx + i] = v;
        }
        const float rx = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)g.k + g.eps);
        for (int i = t; i < g.kpad; i += 256) {
            const float v = i < g.k ? xs[i] * rx * g.g[i] : 0.0f;
            xs[i] = v;
            if (blockIdx.x == 0 && g.h_out && i < g.k) g.h_out[(size_t)tok * g.ldh + i] = v;
        }
    } else {
        for (int i = t; i < g.kpad; i += 256) xs[i] = i < g.k ? x[i] : 0.0f;
    }
    __syncthreads();
    // ---- the products
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.0f;
    auto dot = [&](int c, const uint4 (&u)[R]) {
        float xv[CE];
#pragma unroll
        for (int q = 0; q < CE / 4; q++) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(xs + c * CE + q * 4);
#pragma unroll
            for (int e = 0; e < 4; e++) xv[q * 4 + e] = v[e];
        }
#pragma unroll
        for (int r = 0; r < R; r++) {
            float wv[CE];
            Chunk<ET>::unpack(u[r], wv);
#pragma unroll
            for (int e = 0; e < CE; e++) acc[r] = fma_f(wv[e], xv[e], acc[r]);
        }
    };
#pragma unroll
    for (int s = 0; s < S; s++) {
        const int c = s * 256 + t;
        if (c < nchunk) {
            uint4 u[R];
#pragma unroll
            for (int r = 0; r < R; r++) u[r] = pre[r][s];
            dot(c, u);
        }
    }
    for (int c = S * 256 + t; c < nchunk; c += 256) {
        uint4 u[R];
#pragma unroll
        for (int r = 0; r < R; r++) u[r] = *reinterpret_cast<const uint4*>(w + (size_t)min(row0 + r, g.n - 1) * g.kpad + c * CE);
        dot(c, u);
    }
    multi_sum_step<R, 1>(acc, lane);
    if (lane < R) red[wave * R + multi_row<R>(lane)] = acc[0];
    __syncthreads();
    if (t < R) {
        const int row = row0 + t;
        float v[2];
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int r = i == 0 ? t : min(t + 1, R - 1);
            v[i] = (red[r] + red[R + r]) + (red[2 * R + r] + red[3 * R + r]);
        }
        if (row < g.n) {
            const size_t o = blockIdx.y;
            if (row >= g.n_split) g.out32[o * g.ldo32 + row - g.n_split] = v[0];
            else if (!g.glu) g.out[o * g.ldo + row] = v[0];
            else if ((row & 1) == 0) g.out[o * g.ldo + (row >> 1)] = clamped_glu_f(v[0], v[1], g.limit);
        }
    }
}

template <typename ET, int R, int S>
static int launch_gemv_rs(const GemvArgs& g, int pro, int rows_y, hipStream_t st) {
    const dim3 grid((g.n + R - 1) / R, rows_y);
    const size_t lds = (size_t)g.kpad * sizeof(float);
    if (pro == 0) gemv_float_kernel<ET, R, S, 0><<<grid, 256, lds, st>>>(g);
    else if (pro == 1) gemv_float_kernel<ET, R, S, 1><<<grid, 256, lds, st>>>(g);
    else gemv_float_kernel<ET, R, S, 2><<<grid, 256, lds, st>>>(g);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

template <typename ET>
int gemv_float(const GemvArgs& g, int pro, int tokens, hipStream_t st) {
    FX_REQUIRE(g.w && g.x && g.n > 0 && g.k > 0 && g.kpad >= g.k && g.kpad % kKPad == 0 && tokens > 0, "gemv_float: n=%d k=%d", g.n, g.k);
    FX_REQUIRE(g.kpad <= 15360, "gemv_float: k=%d beyond 15360 (the vector is held in LDS)", g.k);
    FX_REQUIRE(pro != 2 || (g.experts > 0 && g.experts <= kMaxExperts && g.top > 0 && g.top <= kMaxTop && g.top <= g.experts),
               "gemv_float: %d experts, top %d (at most %d, %d)", g.experts, g.top, kMaxExperts, kMaxTop);
    const int per = 256 * Chunk<ET>::N, steps = (g.kpad + per - 1) / per;
    const int rows_y = pro == 2 ? tokens * g.top : tokens;
    auto wgs = [&](int r) { return (g.n + r - 1) / r * rows_y; };
    if (steps == 1) {
        if (wgs(16) >= 512) return launch_gemv_rs<ET, 16, 1>(g, pro, rows_y, st);
        if (wgs(8) >= 384) return launch_gemv_rs<ET, 8, 1>(g, pro, rows_y, st);
        return launch_gemv_rs<ET, 4, 1>(g, pro, rows_y, st);
    }
    if (steps == 2) {
        if (wgs(8) >= 384) return launch_gemv_rs<ET, 8, 2>(g, pro, rows_y, st);
        return launch_gemv_rs<ET, 4, 2>(g, pro, rows_y, st);
    }
    return launch_gemv_rs<ET, 4, 4>(g, pro, rows_y, st);
}
template int gemv_float<bf16_t>(const GemvArgs&, int, int, hipStream_t);
template int gemv_float<float>(const GemvArgs&, int, int, hipStream_t);

// Down projections of the chosen experts and of the shared one, summed with their weights.  The sources lie one after
// the other in a list of 16-byte pieces, which the threads walk together; R = 4 output rows per workgroup.
template <typename ET>
__global__ __launch_bounds__(256) void moe_down_kernel(MoeDownArgs a) {
    constexpr int CE = Chunk<ET>::N, R = 4;
    __shared__ float red[4 * R];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, tok = blockIdx.y, row0 = blockIdx.x * R;
    const int ce = a.kpad / CE, cs = a.ws ? a.ks_pad / CE : 0, total = a.top * ce + cs;
    float acc[R] = {0.0f, 0.0f, 0.0f, 0.0f};
    float sg = 0.0f;
    if (a.ws) sg = sigmoid_f(a.route[(size_t)tok * a.ld_route + a.experts]);
#pragma unroll 4
    for (int it = t; it < total; it += 256) {
        const bool sh = it >= a.top * ce;
        const int slot = sh ? 0 : it / ce, c = sh ? it - a.top * ce : it - slot * ce;
        const int kp = sh ? a.ks_pad : a.kpad, kk = sh ? a.ks : a.k;
        const ET* w = sh ? static_cast<const ET*>(a.ws) : static_cast<const ET*>(a.w) + (size_t)a.pick[tok * a.top + slot] * a.w_stride;
        const float wt = sh ? sg : a.pick_w[tok * a.top + slot];
        const float* h = sh ? a.hs + (size_t)tok * a.ldhs : a.h + (size_t)(tok * a.top + slot) * a.ldh;
        uint4 u[R];
#pragma unroll
        for (int r = 0; r < R; r++) u[r] = *reinterpret_cast<const uint4*>(w + (size_t)min(row0 + r, a.n - 1) * kp + c * CE);
        float xv[CE];
#pragma unroll
        for (int e = 0; e < CE; e++) xv[e] = c * CE + e < kk ? h[c * CE + e] : 0.0f;
#pragma unroll
        for (int r = 0; r < R; r++) {
            float wv[CE], s = 0.0f;
            Chunk<ET>::unpack(u[r], wv);
#pragma unroll
            for (int e = 0; e < CE; e++) s = fma_f(wv[e], xv[e], s);
            acc[r] = fma_f(wt, s, acc[r]);
        }
    }
    multi_sum_step<R, 1>(acc, lane);
    if (lane < R) red[wave * R + multi_row<R>(lane)] = acc[0];
    __syncthreads();
    if (t < R && row0 + t < a.n)
        a.y[(size_t)tok * a.ldy + row0 + t] = (red[t] + red[R + t]) + (red[2 * R + t] + red[3 * R + t]);
}

template <typename ET>
int moe_down_small(const MoeDownArgs& a, int tokens, hipStream_t st) {
    FX_REQUIRE(a.w && a.h && a.pick && a.pick_w && a.y && a.n > 0 && tokens > 0, "moe_down: null pointer");
    moe_down_kernel<ET><<<dim3((a.n + 3) / 4, tokens), 256, 0, st>>>(a);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int moe_down_small<bf16_t>(const MoeDownArgs&, int, hipStream_t);
template int moe_down_small<float>(const MoeDownArgs&, int, hipStream_t);

// ---- the plan of a mixture over many rows --------------------------------------------------------------------------
static __global__ __launch_bounds__(256) void moe_clear_kernel(int* counts, int n) {
    for (int i = threadIdx.x; i < n; i += 256) counts[i] = 0;
}
static __global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ route, int ld, int rows, int experts, int top,
                                                               int* __restrict__ pick, float* __restrict__ pick_w, int* __restrict__ counts) {
    __shared__ int sel[4][kMaxTop];
    __shared__ float wt[4][kMaxTop];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, row = blockIdx.x * 4 + wave;
    if (row >= rows) return;
    route_wave(route + (size_t)row * ld, experts, top, sel[wave], wt[wave]);
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    if (lane < top) {
        const int e = sel[wave][lane];
        pick[row * top + lane] = e;
        pick_w[row * top + lane] = wt[wave][lane];
        atomicAdd(&counts[e], 1);
    }
}
// Place every (row, choice) in its expert's run; block 0 also cuts the runs into tiles.
static __global__ __launch_bounds__(256) void moe_place_kernel(int rows, int experts, int top, int tile_rows, const int* __restrict__ pick,
                                                               int* __restrict__ counts, int* __restrict__ pos_of, int* __restrict__ row_src,
                                                               int4* __restrict__ tiles, int* __restrict__ n_tiles) {
    __shared__ int first[kMaxExperts + 1], tile0[kMaxExperts + 1];
    __shared__ int part[256], part_t[256];
    const int t = threadIdx.x;
    const int per = (experts + 255) / 256;
    int s = 0, st = 0;
    for (int i = 0; i < per; i++) {
        const int e = t * per + i;
        if (e < experts) { s += counts[e]; st += (counts[e] + tile_rows - 1) / tile_rows; }
    }
    part[t] = s; part_t[t] = st;
    __syncthreads();
    for (int m = 1; m < 256; m <<= 1) {                   // inclusive scan
        const int a = t >= m ? part[t - m] : 0, b = t >= m ? part_t[t - m] : 0;
        __syncthreads();
        part[t] += a; part_t[t] += b;
        __syncthreads();
    }
    int o = part[t] - s, ot = part_t[t] - st;
    for (int i = 0; i < per; i++) {
        const int e = t * per + i;
        if (e < experts) { first[e] = o; tile0[e] = ot; o += counts[e]; ot += (counts[e] + tile_rows - 1) / tile_rows; }
    }
    __syncthreads();
    const int idx = blockIdx.x * 256 + t;
    if (idx < rows * top) {
        const int e = pick[idx];
        const int pos = first[e] + atomicAdd(&counts[experts + e], 1);
        pos_of[idx] = pos;
        row_src[pos] = idx / top;
    }
    if (blockIdx.x == 0) {
        for (int e = t; e < experts; e += 256) {
            const int n = counts[e];
            for (int i = 0; i * tile_rows < n; i++)
                tiles[tile0[e] + i] = make_int4(e, first[e] + i * tile_rows, first[e] + min(n, (i + 1) * tile_rows), 0);
        }
        if (t == 0) n_tiles[0] = part_t[255];
    }
}

int moe_plan(const float* route, int ld_route, int rows, int experts, int top, int tile_rows, const MoePlan& p, hipStream_t st) {
    FX_REQUIRE(experts > 0 && experts <= kMaxExperts && top > 0 && top <= kMaxTop && top <= experts, "moe_plan: %d experts, top %d (at most %d, %d)",
               experts, top, kMaxExperts, kMaxTop);
    moe_clear_kernel<<<1, 256, 0, st>>>(p.counts, 2 * experts);
    moe_route_kernel<<<(rows + 3) / 4, 256, 0, st>>>(route, ld_route, rows, experts, top, p.pick, p.pick_w, p.counts);
    moe_place_kernel<<<(rows * top + 255) / 256, 256, 0, st>>>(rows, experts, top, tile_rows, p.pick, p.counts, p.pos_of, p.row_src, p.tiles, p.n_tiles);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

}  // namespace fx
