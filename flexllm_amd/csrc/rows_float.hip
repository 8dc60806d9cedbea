// Row kernels of the floating-point layers: weight packing, embedding rows, and the fused
// residual + norm after a sublayer + norm before the next one (with the mixture's weighted sum in front).
#include "float_ops.h"

namespace fx {

// dst row i*row_step + row_off = source row i, widened or copied, zero beyond k (rows are kpad long)
template <typename ET>
__global__ __launch_bounds__(256) void pack_rows_kernel(const bf16_t* __restrict__ src, ET* __restrict__ dst, int k, int kpad, int row_step, int row_off) {
    const bf16_t* s = src + (size_t)blockIdx.x * k;
    ET* d = dst + ((size_t)blockIdx.x * row_step + row_off) * kpad;
    for (int i = threadIdx.x; i < kpad; i += 256) d[i] = i < k ? (ET)s[i] : (ET)0.0f;
}
template <typename ET>
int pack_rows(const bf16_t* src, ET* dst, int n, int k, int kpad, int row_step, int row_off, hipStream_t st) {
    FX_REQUIRE(src && dst && n > 0 && k > 0 && kpad >= k, "pack_rows: n=%d k=%d", n, k);
    pack_rows_kernel<ET><<<n, 256, 0, st>>>(src, dst, k, kpad, row_step, row_off);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int pack_rows<bf16_t>(const bf16_t*, bf16_t*, int, int, int, int, int, hipStream_t);
template int pack_rows<float>(const bf16_t*, float*, int, int, int, int, int, hipStream_t);

static __global__ __launch_bounds__(256) void widen_rows_kernel(const bf16_t* __restrict__ src, float* __restrict__ dst, int n, float add) {
    for (int i = blockIdx.x * 256 + threadIdx.x; i < n; i += gridDim.x * 256) dst[i] = (float)src[i] + add;
}
int widen_rows(const bf16_t* src, float* dst, int n, float add, hipStream_t st) {
    FX_REQUIRE(src && dst && n > 0, "widen_rows: n=%d", n);
    widen_rows_kernel<<<(n + 255) / 256, 256, 0, st>>>(src, dst, n, add);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

// Ids outside [0, vocab) are replaced by 0 and reported through *err = 2, as in embed_rows_kernel.
static __global__ __launch_bounds__(256) void embed_bf16_kernel(const bf16_t* __restrict__ table, float scale, const int* __restrict__ tokens, float* __restrict__ x,
                                                                int width, int vocab, int* __restrict__ err) {
    int tk = tokens[blockIdx.x];
    if ((unsigned)tk >= (unsigned)vocab) {
        if (err && threadIdx.x == 0) err[0] = 2;
        tk = 0;
    }
    const bf16_t* s = table + (size_t)tk * width;
    for (int i = threadIdx.x; i < width; i += 256) x[(size_t)blockIdx.x * width + i] = (float)s[i] * scale;
}
int embed_rows_bf16(const bf16_t* table, float scale, const int* tokens, int n, float* x, int width, int vocab, int* err, hipStream_t st) {
    embed_bf16_kernel<<<n, 256, 0, st>>>(table, scale, tokens, x, width, vocab, err);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

static __global__ void put_state_kernel(int* state, int pos, int step) { state[0] = pos; state[1] = step; }
static __global__ void advance_kernel(int* state, int n) { state[0] += n; }
int set_state_launch(int* state, int pos, int step, hipStream_t st) {
    put_state_kernel<<<1, 1, 0, st>>>(state, pos, step);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
int advance_launch(int* state, int n, hipStream_t st) {
    advance_kernel<<<1, 1, 0, st>>>(state, n);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

// One workgroup per row; the row stays in LDS between the two norms.
template <typename ET>
__global__ __launch_bounds__(256) void norm_rows_kernel(RowArgs a) {
    extern __shared__ float row[];
    __shared__ float red[4];
    const int t = threadIdx.x, r = blockIdx.x;
    const float* x = a.x + (size_t)(a.rows_src ? a.rows_src[r] : r) * a.width;
    float* x_new = (a.x_new ? a.x_new : a.x) + (size_t)r * a.width;
    const bool mix = a.ys != nullptr, have_y = a.y || mix;
    if (have_y || a.x0) {
        float sg = 1.0f;
        if (mix && a.y) sg = sigmoid_f(a.route[(size_t)r * a.ld_route + a.experts]);
        float ss = 0.0f;
        for (int i = t; i < a.width; i += 256) {
            float v = 0.0f;
            if (mix) {
                for (int k = 0; k < a.top; k++) v = fma_f(a.pick_w[r * a.top + k], a.ys[(size_t)a.pos_of[r * a.top + k] * a.ldy + i], v);
                if (a.y) v = fma_f(sg, a.y[(size_t)r * a.ldy + i], v);
            } else if (a.y) {
                v = a.y[(size_t)r * a.ldy + i];
            }
            row[i] = v;
            ss = fma_f(v, v, ss);
        }
        const bool post = have_y && a.gb;
        const float rs = post ? 1.0f / sqrtf(block_sum<4>(ss, red) / (float)a.width + a.eps) : 1.0f;
        for (int i = t; i < a.width; i += 256) {
            float v = x[i] + (post ? row[i] * rs * a.gb[i] : row[i]);
            if (a.x0) v += a.x0[(size_t)r * a.width + i];
            row[i] = v;
            if (!a.rows_src) x_new[i] = v;
        }
    } else {
        for (int i = t; i < a.width; i += 256) row[i] = x[i];
    }
    if (!a.h) return;
    float ss = 0.0f;
    for (int i = t; i < a.width; i += 256) ss = fma_f(row[i], row[i], ss);
    const float rx = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)a.width + a.eps);
    if (a.h_f32) {
        float* h = static_cast<float*>(a.h) + (size_t)r * a.ldh;
        for (int i = t; i < a.width; i += 256) h[i] = row[i] * rx * a.g[i];
    } else {
        ET* h = static_cast<ET*>(a.h) + (size_t)r * a.ldh;
        for (int i = t; i < a.ldh; i += 256) h[i] = i < a.width ? (ET)(row[i] * rx * a.g[i]) : (ET)0.0f;
    }
}

// The same for widths that are a multiple of 4 and at most 256 * 4 * V: the row stays in registers, 16-byte accesses.
template <typename ET, int V>
__global__ __launch_bounds__(256) void norm_rows_vec_kernel(RowArgs a) {
    __shared__ float red[4];
    const int t = threadIdx.x, r = blockIdx.x, n4 = a.width >> 2;
    const float* x = a.x + (size_t)(a.rows_src ? a.rows_src[r] : r) * a.width;
    float* x_new = (a.x_new ? a.x_new : a.x) + (size_t)r * a.width;
    const bool mix = a.ys != nullptr, have_y = a.y || mix;
    f32x4 v[V];
#pragma unroll
    for (int i = 0; i < V; i++) {
        const int c = t + i * 256;
        v[i] = c < n4 ? *reinterpret_cast<const f32x4*>(x + c * 4) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
    if (have_y || a.x0) {
        f32x4 y[V];
        float ss = 0.0f, sg = 1.0f;
        if (mix && a.y) sg = sigmoid_f(a.route[(size_t)r * a.ld_route + a.experts]);
#pragma unroll
        for (int i = 0; i < V; i++) {
            const int c = t + i * 256;
            y[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            if (c < n4) {
                if (mix) {
                    for (int k = 0; k < a.top; k++) {
                        const float w = a.pick_w[r * a.top + k];
                        const f32x4 u = *reinterpret_cast<const f32x4*>(a.ys + (size_t)a.pos_of[r * a.top + k] * a.ldy + c * 4);
#pragma unroll
                        for (int e = 0; e < 4; e++) y[i][e] = fma_f(w, u[e], y[i][e]);
                    }
                    if (a.y) {
                        const f32x4 u = *reinterpret_cast<const f32x4*>(a.y + (size_t)r * a.ldy + c * 4);
#pragma unroll
                        for (int e = 0; e < 4; e++) y[i][e] = fma_f(sg, u[e], y[i][e]);
                    }
                } else if (a.y) {
                    y[i] = *reinterpret_cast<const f32x4*>(a.y + (size_t)r * a.ldy + c * 4);
                }
            }
#pragma unroll
            for (int e = 0; e < 4; e++) ss = fma_f(y[i][e], y[i][e], ss);
        }
        const bool post = have_y && a.gb;
        const float rs = post ? 1.0f / sqrtf(block_sum<4>(ss, red) / (float)a.width + a.eps) : 1.0f;
#pragma unroll
        for (int i = 0; i < V; i++) {
            const int c = t + i * 256;
            if (c >= n4) continue;
            if (post) {
                const f32x4 gb = *reinterpret_cast<const f32x4*>(a.gb + c * 4);
#pragma unroll
                for (int e = 0; e < 4; e++) v[i][e] = v[i][e] + y[i][e] * rs * gb[e];
            } else {
#pragma unroll
                for (int e = 0; e < 4; e++) v[i][e] = v[i][e] + y[i][e];
            }
            if (a.x0) {
                const f32x4 u = *reinterpret_cast<const f32x4*>(a.x0 + (size_t)r * a.width + c * 4);
#pragma unroll
                for (int e = 0; e < 4; e++) v[i][e] += u[e];
            }
            if (!a.rows_src) *reinterpret_cast<f32x4*>(x_new + c * 4) = v[i];
        }
    }
    if (!a.h) return;
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < V; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) ss = fma_f(v[i][e], v[i][e], ss);
    const float rx = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)a.width + a.eps);
#pragma unroll
    for (int i = 0; i < V; i++) {
        const int c = t + i * 256;
        if (c >= n4) continue;
        const f32x4 g = *reinterpret_cast<const f32x4*>(a.g + c * 4);
        f32x4 o;
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] = v[i][e] * rx * g[e];
        if (a.h_f32 || std::is_same<ET, float>::value) {
            *reinterpret_cast<f32x4*>(static_cast<float*>(a.h) + (size_t)r * a.ldh + c * 4) = o;
        } else {
            bf16x4 b;
#pragma unroll
            for (int e = 0; e < 4; e++) b[e] = (bf16_t)o[e];
            *reinterpret_cast<bf16x4*>(static_cast<bf16_t*>(a.h) + (size_t)r * a.ldh + c * 4) = b;
        }
    }
}

template <typename ET>
int norm_rows(const RowArgs& a, hipStream_t st) {
    FX_REQUIRE(a.x && a.rows > 0 && a.width > 0 && a.width <= 16384 && (!a.h || (a.g && a.ldh >= a.width)), "norm_rows: rows=%d width=%d", a.rows, a.width);
    const bool vec = a.width % 4 == 0 && a.ldy % 4 == 0 && a.ldh % 4 == 0;
    if (vec && a.width <= 1024) norm_rows_vec_kernel<ET, 1><<<a.rows, 256, 0, st>>>(a);
    else if (vec && a.width <= 2048) norm_rows_vec_kernel<ET, 2><<<a.rows, 256, 0, st>>>(a);
    else if (vec && a.width <= 4096) norm_rows_vec_kernel<ET, 4><<<a.rows, 256, 0, st>>>(a);
    else norm_rows_kernel<ET><<<a.rows, 256, a.width * sizeof(float), st>>>(a);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}
template int norm_rows<bf16_t>(const RowArgs&, hipStream_t);
template int norm_rows<float>(const RowArgs&, hipStream_t);

}  // namespace fx
