// Element types of the floating-point layers: weights and activations in bfloat16 (served precision) or in float32.
// Kernels are templates over the element type ET; sums, norms, scores and states are float32 in both.
#pragma once
#include "common.h"
#include <type_traits>

namespace fx {

using bf16_t = __bf16;
using bf16x8 = __bf16 __attribute__((ext_vector_type(8)));
using bf16x4 = __bf16 __attribute__((ext_vector_type(4)));
using f32x16 = float __attribute__((ext_vector_type(16)));

constexpr int kKPad = 64;                                 // rows of weights and activations are padded to 64 elements
__host__ __device__ constexpr int pad_k(int k) { return (k + kKPad - 1) / kKPad * kKPad; }

template <typename ET> struct Chunk;                      // one 16-byte piece of a row
template <> struct Chunk<bf16_t> {
    static constexpr int N = 8;
    __device__ static __forceinline__ void unpack(const uint4& u, float (&v)[8]) {
        const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
        for (int i = 0; i < 4; i++) {
            v[2 * i] = __int_as_float((int)(w[i] << 16));
            v[2 * i + 1] = __int_as_float((int)(w[i] & 0xFFFF0000u));
        }
    }
};
template <> struct Chunk<float> {
    static constexpr int N = 4;
    __device__ static __forceinline__ void unpack(const uint4& u, float (&v)[4]) {
        v[0] = __int_as_float((int)u.x); v[1] = __int_as_float((int)u.y);
        v[2] = __int_as_float((int)u.z); v[3] = __int_as_float((int)u.w);
    }
};

__device__ __forceinline__ float fma_f(float a, float b, float c) { return __builtin_fmaf(a, b, c); }
__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + exp_f(-v)); }

// log(sigmoid(z)) = min(z, 0) - log(1 + exp(-|z|)): no cancellation and no overflow for any z
__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.0f) - log1pf(exp_f(-fabsf(z))); }

// Gated linear unit with clamped inputs: g = min(gate, limit), u = clamp(up, -limit, limit), g sigmoid(1.702 g) (u + 1)
__device__ __forceinline__ float clamped_glu_f(float gate, float up, float limit) {
    const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
    return g * sigmoid_f(1.702f * g) * (u + 1.0f);
}

// Gated linear unit with the tanh form of gelu: 0.5 z (1 + tanh(u)) = z sigmoid(2u), u = sqrt(2/pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_glu_f(float gate, float up) {
    const float u = 0.7978845608028654f * fma_f(0.044715f * gate * gate, gate, gate);
    return gate * sigmoid_f(2.0f * u) * up;
}

// The units that the linears can apply to gate/up pairs (GemmArgs::glu, GemvArgs::glu; 0: none)
enum GluKind { kGluClamped = 1, kGluGelu = 2 };
__device__ __forceinline__ float glu_f(int kind, float gate, float up, float limit) {
    return kind == kGluGelu ? gelu_glu_f(gate, up) : clamped_glu_f(gate, up, limit);
}

// R sums over the 64 lanes of a wave at once: every halving step hands half of the values to the partner lane, so the
// total is 2R moves instead of 6R.  Afterwards lane l (l < R) holds the sum of row multi_row<R>(l).
template <int R, int MASK>
__device__ __forceinline__ void multi_sum_step(float* v, int lane) {
    if constexpr (R > 1) {
        const bool up = lane & MASK;
#pragma unroll
        for (int i = 0; i < R / 2; i++) {
            const float keep = up ? v[i + R / 2] : v[i], send = up ? v[i] : v[i + R / 2];
            v[i] = keep + lane_xor_f<MASK>(send);
        }
    } else {
        v[0] += lane_xor_f<MASK>(v[0]);
    }
    if constexpr (MASK < 32) multi_sum_step<(R > 1 ? R / 2 : 1), MASK * 2>(v, lane);
}
template <int R>
__device__ __forceinline__ int multi_row(int lane) {
    int row = 0;
#pragma unroll
    for (int m = 1, h = R / 2; h >= 1; m *= 2, h /= 2)
        if (lane & m) row += h;
    return row;
}

}  // namespace fx
