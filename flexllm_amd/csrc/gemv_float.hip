// Linears of one token: y = W h with W of ET (bfloat16 or float32) streamed once, h float32 in LDS.
//
// A workgroup of 256 threads walks groups of R weight rows; thread t reads 16-byte pieces t, t + 256, ... of each row.
// The first two groups are requested before the prologue (residual, norms) runs, so that its latency lies under the weight
// stream, and two groups stay in flight after that.  The R sums are reduced together (multi_sum_step).
#include "float_ops.h"

namespace fx {

constexpr int kMaxExperts = 1024, kMaxTop = 32;

// Expert choice of one token by one wave: softmax over the router outputs, the `top` largest (ties: lower index), their
// weights divided by their sum.  Lane k < top gets choice k and its weight.  NE: 64-expert pieces (experts <= 64 NE).
template <int NE>
__device__ __forceinline__ void route_wave_n(const float* __restrict__ z, int experts, int top, int& pick, float& weight) {
    const int lane = threadIdx.x & 63;
    float v[NE];
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < NE; i++) {
        v[i] = i * 64 + lane < experts ? z[i * 64 + lane] : -INFINITY;
        mx = fmaxf(mx, v[i]);
    }
    mx = wave_max(mx);
    float den = 0.0f;
#pragma unroll
    for (int i = 0; i < NE; i++) {
        v[i] = i * 64 + lane < experts ? exp_f<false>(v[i] - mx) : -1.0f;
        den += fmaxf(v[i], 0.0f);
    }
    den = wave_sum(den);
    float sum = 0.0f;
    pick = 0;
    weight = 0.0f;
    for (int k = 0; k < top; k++) {
        float best = v[0];
#pragma unroll
        for (int i = 1; i < NE; i++) best = fmaxf(best, v[i]);
        best = wave_max(best);
        int bi = -1;                                      // lowest index that holds the maximum
#pragma unroll
        for (int i = 0; i < NE; i++) {
            const unsigned long long hit = __ballot(v[i] == best);
            if (bi < 0 && hit) {
                const int l = __builtin_ctzll(hit);
                bi = i * 64 + l;
                if (lane == l) v[i] = -1.0f;
            }
        }
        const float s = best / den;
        sum += s;
        if (lane == k) { pick = bi; weight = s; }
    }
    weight = weight / (sum + 1e-20f);
}
__device__ __forceinline__ void route_wave(const float* __restrict__ z, int experts, int top, int& pick, float& weight) {
    if (experts <= 64) route_wave_n<1>(z, experts, top, pick, weight);
    else if (experts <= 256) route_wave_n<4>(z, experts, top, pick, weight);
    else route_wave_n<kMaxExperts / 64>(z, experts, top, pick, weight);
}

// VEC: the prologue keeps its vectors in registers as float4 (k a multiple of 4, at most what the S pieces per thread cover);
// else any k, through LDS.
template <typename ET, int R, int S, int PRO, bool VEC>
__global__ __launch_bounds__(256) void gemv_float_kernel(GemvArgs g) {
    constexpr int CE = Chunk<ET>::N;
    extern __shared__ __attribute__((aligned(16))) float xs[];     // [kpad] the vector
    __shared__ float red[2][4 * R];
    __shared__ float nred[4];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int tok = PRO == 2 ? blockIdx.y / g.top : blockIdx.y;
    const ET* w = static_cast<const ET*>(g.w);
    const float* x = g.x + (size_t)tok * g.ldx;
    // ---- requests for the vector go out first: loads return in order, and the weights behind them are a long stream
    constexpr int Q = VEC ? S * CE / 4 : 1;               // float4 per thread
    f32x4 xv[Q], yv[Q], gb[Q], gv[Q];
    const int k4 = g.k >> 2;
    const bool have_y = PRO == 1 && g.y != nullptr, post = have_y && g.gb != nullptr;
    // gb holds the weight of the norm after the sublayer, or where there is none the other vector to add
    const float* extra = post ? g.gb : g.x0 ? g.x0 + (size_t)tok * g.ldx : nullptr;
    if constexpr (VEC) {
        const f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
        const float* y = g.y + (size_t)tok * g.ldy;
#pragma unroll
        for (int i = 0; i < Q; i++) {
            const int c = t + 256 * i;
            const bool in = c < k4;
            if constexpr (PRO == 1) yv[i] = in && have_y ? *reinterpret_cast<const f32x4*>(y + 4 * c) : zero;
            xv[i] = in ? *reinterpret_cast<const f32x4*>(x + 4 * c) : zero;
            if constexpr (PRO == 1) {
                gb[i] = in && extra ? *reinterpret_cast<const f32x4*>(extra + 4 * c) : zero;
                gv[i] = in ? *reinterpret_cast<const f32x4*>(g.g + 4 * c) : zero;
            }
        }
        __builtin_amdgcn_sched_barrier(0);
    }
    if constexpr (PRO == 2) {
        int pick;                                         // every wave chooses for itself: no barrier before the weights
        float weight;
        route_wave(g.route + (size_t)tok * g.ld_route, g.experts, g.top, pick, weight);
        const int slot = blockIdx.y % g.top;
        w += (size_t)__builtin_amdgcn_readlane(pick, slot) * g.w_stride;
        if (blockIdx.x == 0 && t == slot) { g.pick[blockIdx.y] = pick; g.pick_w[blockIdx.y] = weight; }
    }
    const int nchunk = g.kpad / CE;                       // 16-byte pieces of a row
    const int ng = (g.n + R - 1) / R, G = gridDim.x;      // groups of R rows, dealt to the workgroups in turn
    i32x4 buf[2][R][S];
    auto piece = [&](int row, int c) { return *reinterpret_cast<const i32x4*>(w + (size_t)min(row, g.n - 1) * g.kpad + c * CE); };
    auto load = [&](int b, int grp) {
#pragma unroll
        for (int r = 0; r < R; r++)
#pragma unroll
            for (int s = 0; s < S; s++) {
                const int c = s * 256 + t;
                buf[b][r][s] = c < nchunk ? piece(grp * R + r, c) : i32x4{0, 0, 0, 0};
            }
    };
    const int g0 = blockIdx.x;
    load(0, g0);
    if (g0 + G < ng) load(1, g0 + G);
    __builtin_amdgcn_sched_barrier(0);
    // ---- the vector
    if constexpr (PRO == 1 && VEC) {
        float rs = 0.0f;
        if (post) {
            float ss = 0.0f;
#pragma unroll
            for (int i = 0; i < Q; i++)
#pragma unroll
                for (int e = 0; e < 4; e++) ss = fma_f(yv[i][e], yv[i][e], ss);
            rs = 1.0f / sqrtf(block_sum<4>(ss, nred) / (float)g.k + g.eps);
        }
        float ss = 0.0f;
#pragma unroll
        for (int i = 0; i < Q; i++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                xv[i][e] = post ? xv[i][e] + yv[i][e] * rs * gb[i][e] : xv[i][e] + yv[i][e] + gb[i][e];
                ss = fma_f(xv[i][e], xv[i][e], ss);
            }
        const float rx = 1.0f / sqrtf(block_sum<4>(ss, nred) / (float)g.k + g.eps);
#pragma unroll
        for (int i = 0; i < Q; i++) {
            const int c = t + 256 * i;
            f32x4 h;
#pragma unroll
            for (int e = 0; e < 4; e++) h[e] = xv[i][e] * rx * gv[i][e];
            if (4 * c < g.kpad) *reinterpret_cast<f32x4*>(xs + 4 * c) = h;
            if (blockIdx.x == 0 && c < k4) {
                if (g.x_new) *reinterpret_cast<f32x4*>(g.x_new + (size_t)tok * g.ldx + 4 * c) = xv[i];
                if (g.h_out) *reinterpret_cast<f32x4*>(g.h_out + (size_t)tok * g.ldh + 4 * c) = h;
            }
        }
    } else if constexpr (PRO == 1) {
        float rs = 0.0f;
        if (have_y) {
            const float* y = g.y + (size_t)tok * g.ldy;
            float ss = 0.0f;
            for (int i = t; i < g.k; i += 256) { const float v = y[i]; xs[i] = v; ss = fma_f(v, v, ss); }
            if (post) rs = 1.0f / sqrtf(block_sum<4>(ss, nred) / (float)g.k + g.eps);
        }
        float ss = 0.0f;
        for (int i = t; i < g.k; i += 256) {
            float v = x[i];
            if (post) v = v + xs[i] * rs * extra[i];
            else {
                if (have_y) v += xs[i];
                if (extra) v += extra[i];
            }
            xs[i] = v;
            ss = fma_f(v, v, ss);
            if (blockIdx.x == 0 && g.x_new) g.x_new[(size_t)tok * g.ldx + i] = v;
        }
        const float rx = 1.0f / sqrtf(block_sum<4>(ss, nred) / (float)g.k + g.eps);
        for (int i = t; i < g.kpad; i += 256) {
            const float v = i < g.k ? xs[i] * rx * g.g[i] : 0.0f;
            xs[i] = v;
            if (blockIdx.x == 0 && g.h_out && i < g.k) g.h_out[(size_t)tok * g.ldh + i] = v;
        }
    } else if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < Q; i++)
            if (4 * (t + 256 * i) < g.kpad) *reinterpret_cast<f32x4*>(xs + 4 * (t + 256 * i)) = xv[i];
    } else {
        for (int i = t; i < g.kpad; i += 256) xs[i] = i < g.k ? x[i] : 0.0f;
    }
    __syncthreads();
    // ---- the products
    auto dot = [&](int c, const i32x4& u, float& acc) {
        float wv[CE];
        Chunk<ET>::unpack(make_uint4(u[0], u[1], u[2], u[3]), wv);
#pragma unroll
        for (int q = 0; q < CE / 4; q++) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(xs + c * CE + q * 4);
#pragma unroll
            for (int e = 0; e < 4; e++) acc = fma_f(wv[q * 4 + e], v[e], acc);
        }
    };
    auto process = [&](int b, int grp) {
        float acc[R];
        float bias[2] = {0.0f, 0.0f};                     // of the rows that this thread hands out below
        if (g.bias && t < R) {
            bias[0] = g.bias[min(grp * R + t, g.n - 1)];
            bias[1] = g.bias[min(grp * R + t + 1, g.n - 1)];
        }
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = 0.0f;
#pragma unroll
        for (int s = 0; s < S; s++) {
            const int c = min(s * 256 + t, nchunk - 1);   // pieces beyond the row were filled with zeros
#pragma unroll
            for (int r = 0; r < R; r++) dot(c, buf[b][r][s], acc[r]);
        }
        for (int c = S * 256 + t; c < nchunk; c += 256)
#pragma unroll
            for (int r = 0; r < R; r++) dot(c, piece(grp * R + r, c), acc[r]);
        multi_sum_step<R, 1>(acc, lane);
        if (lane < R) red[b][wave * R + multi_row<R>(lane)] = acc[0];
        __syncthreads();                                  // red alternates with the buffer: one barrier per group is enough
        if (t < R) {
            const int row = grp * R + t;
            float v[2];
#pragma unroll
            for (int i = 0; i < 2; i++) {
                const int r = min(t + i, R - 1);
                v[i] = (red[b][r] + red[b][R + r]) + (red[b][2 * R + r] + red[b][3 * R + r]) + bias[i];
            }
            if (row < g.n) {
                const size_t o = blockIdx.y;
                if (row >= g.n_split) g.out32[o * g.ldo32 + row - g.n_split] = v[0];
                else if (!g.glu) g.out[o * g.ldo + row] = v[0];
                else if ((row & 1) == 0) g.out[o * g.ldo + (row >> 1)] = glu_f(g.glu, v[0], v[1], g.limit);
            }
        }
    };
    for (int grp = g0; grp < ng; grp += 2 * G) {
        process(0, grp);
        if (grp + 2 * G < ng) load(0, grp + 2 * G);
        if (grp + G < ng) {
            process(1, grp + G);
            if (grp + 3 * G < ng) load(1, grp + 3 * G);
        }
    }
}

template <typename ET, int R, int S>
static int launch_gemv_rs(const GemvArgs& g, int pro, int rows_y, hipStream_t st) {
    // workgroups that share the chip at a time (two per CU where the vector takes a third of LDS or more); each walks its
    // groups with the next one's weights in flight
    int wgs = (S > 4 ? 512 : 1024) / rows_y;
    if (wgs < 128) wgs = 128;
    const int ng = (g.n + R - 1) / R;
    const dim3 grid(ng < wgs ? ng : wgs, rows_y);
    const size_t lds = (size_t)g.kpad * sizeof(float);
    const bool vec = g.k % 4 == 0 && g.ldx % 4 == 0 && g.ldy % 4 == 0 && g.ldh % 4 == 0 && g.kpad <= 256 * Chunk<ET>::N * S;
#define FX_GEMV(PRO)                                                                               \
    do {                                                                                           \
        if (vec) gemv_float_kernel<ET, R, S, PRO, true><<<grid, 256, lds, st>>>(g);                \
        else gemv_float_kernel<ET, R, S, PRO, false><<<grid, 256, lds, st>>>(g);                   \
    } while (0)
    if (pro == 0) FX_GEMV(0);
    if constexpr (S <= 4) {                               // longer rows: gemv_float asks for the plain linear only
        if (pro == 1) FX_GEMV(1);
        if (pro == 2) FX_GEMV(2);
    }
#undef FX_GEMV
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
    if (steps == 1) {
        if ((g.n + 7) / 8 * rows_y >= 512) return launch_gemv_rs<ET, 8, 1>(g, pro, rows_y, st);
        return launch_gemv_rs<ET, 4, 1>(g, pro, rows_y, st);
    }
    if (steps == 2) return launch_gemv_rs<ET, 4, 2>(g, pro, rows_y, st);
    if (steps > 4 && pro == 0) return launch_gemv_rs<ET, 2, 8>(g, pro, rows_y, st);
    return launch_gemv_rs<ET, 2, 4>(g, pro, rows_y, st);
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
constexpr int kPlanT = 1024, kRouteRows = 32;              // rows per workgroup of the route kernel
static __global__ __launch_bounds__(kPlanT) void moe_route_kernel(const float* __restrict__ route, int ld, int rows, int experts, int top,
                                                                  int* __restrict__ pick, float* __restrict__ pick_w, int* __restrict__ counts) {
    __shared__ int hist[kMaxExperts];
    const int t = threadIdx.x, wave = t >> 6, lane = t & 63;
    for (int e = t; e < experts; e += kPlanT) hist[e] = 0;
    __syncthreads();
    for (int i = 0; i < kRouteRows / (kPlanT / 64); i++) {
        const int row = blockIdx.x * kRouteRows + i * (kPlanT / 64) + wave;
        if (row >= rows) break;
        int e;
        float w;
        route_wave(route + (size_t)row * ld, experts, top, e, w);
        if (lane < top) {
            pick[row * top + lane] = e;
            pick_w[row * top + lane] = w;
            atomicAdd(&hist[e], 1);
        }
    }
    __syncthreads();
    for (int e = t; e < experts; e += kPlanT)
        if (hist[e]) atomicAdd(&counts[e], hist[e]);
}
// Place every (row, choice) in its expert's run: a workgroup reserves room for its entries with one atomic per expert.
// Workgroup 0 also cuts the runs into tiles.
static __global__ __launch_bounds__(kPlanT) void moe_place_kernel(int rows, int experts, int top, int tile_rows, const int* __restrict__ pick,
                                                                  int* __restrict__ counts, int* __restrict__ pos_of, int* __restrict__ row_src,
                                                                  int4* __restrict__ tiles, int* __restrict__ n_tiles) {
    __shared__ int first[kMaxExperts], tile0[kMaxExperts], hist[kMaxExperts];
    __shared__ int part[kPlanT], part_t[kPlanT];
    const int t = threadIdx.x;
    static_assert(kPlanT >= kMaxExperts, "one thread per expert");
    const int n = t < experts ? counts[t] : 0, nt = (n + tile_rows - 1) / tile_rows;
    part[t] = n; part_t[t] = nt;
    if (t < experts) hist[t] = 0;
    __syncthreads();
    for (int m = 1; m < kPlanT; m <<= 1) {                // inclusive scan
        const int a = t >= m ? part[t - m] : 0, b = t >= m ? part_t[t - m] : 0;
        __syncthreads();
        part[t] += a; part_t[t] += b;
        __syncthreads();
    }
    const int idx = blockIdx.x * kPlanT + t, e = idx < rows * top ? pick[idx] : -1;
    const int local = e >= 0 ? atomicAdd(&hist[e], 1) : 0;
    if (t < experts) tile0[t] = part_t[t] - nt;
    __syncthreads();
    if (t < experts) first[t] = part[t] - n + (hist[t] ? atomicAdd(&counts[experts + t], hist[t]) : 0);
    __syncthreads();
    if (e >= 0) {
        const int pos = first[e] + local;
        pos_of[idx] = pos;
        row_src[pos] = idx / top;
    }
    if (blockIdx.x == 0) {
        if (t < experts)
            for (int i = 0; i < nt; i++) tiles[tile0[t] + i] = make_int4(t, part[t] - n + i * tile_rows, part[t] - n + min(n, (i + 1) * tile_rows), 0);
        if (t == 0) n_tiles[0] = part_t[kPlanT - 1];
    }
}

int moe_plan(const float* route, int ld_route, int rows, int experts, int top, int tile_rows, const MoePlan& p, hipStream_t st) {
    FX_REQUIRE(experts > 0 && experts <= kMaxExperts && top > 0 && top <= kMaxTop && top <= experts, "moe_plan: %d experts, top %d (at most %d, %d)",
               experts, top, kMaxExperts, kMaxTop);
    moe_clear_kernel<<<1, 256, 0, st>>>(p.counts, 2 * experts);
    moe_route_kernel<<<(rows + kRouteRows - 1) / kRouteRows, kPlanT, 0, st>>>(route, ld_route, rows, experts, top, p.pick, p.pick_w, p.counts);
    moe_place_kernel<<<(rows * top + kPlanT - 1) / kPlanT, kPlanT, 0, st>>>(rows, experts, top, tile_rows, p.pick, p.counts, p.pos_of, p.row_src, p.tiles, p.n_tiles);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

}  // namespace fx
