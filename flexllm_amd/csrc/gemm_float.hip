// Floating-point GEMMs for prefill: C[m][n] = sum_k A[m][k] * W[n][k], both operands K-contiguous.
//
// bfloat16: the direct-load kernel of the int8 path (gemm_i8.h) on v_mfma_f32_32x32x16_bf16.  A lane's operand is the
// same 16 bytes of a row as in the int8 instruction, so the LDS stage layout, the chunk rotation and the software
// pipeline carry over with K counted in bytes.  Additions: rows of A may be gathered, groups of rows may have a weight
// matrix each (experts), the epilogue adds a bias, splits the columns between an ET and a float32 output and applies the
// gated unit to interleaved gate/up columns.
//
// float32: v_mfma_f32_32x32x2_f32 (full float32 products and sums) on register-staged 64x64 tiles, same epilogue.
#include "float_ops.h"
#include "gemm_i8.h"

namespace fx {

struct GemmTile { int row0, row_end, group; };

// Which tile this workgroup works on: row tiles fastest inside a range of weight columns per XCD, as in gemm_i8_kernel.
template <int BM, int BN>
__device__ __forceinline__ bool gemm_pick_tile(const GemmArgs& g, int tiles_m, int tiles_n, GemmTile& t, int& col0) {
    int tm, tn;
    if ((tiles_n & 7) == 0) {
        const int xcd = blockIdx.x & 7, idx = blockIdx.x >> 3;
        tn = xcd * (tiles_n >> 3) + idx / tiles_m;
        tm = idx % tiles_m;
    } else {
        tm = blockIdx.x % tiles_m;
        tn = blockIdx.x / tiles_m;
    }
    col0 = tn * BN;
    if (g.tiles) {
        if (tm >= g.n_tiles[0]) return false;
        const int4 e = g.tiles[tm];
        t.group = e.x; t.row0 = e.y; t.row_end = e.z;
    } else {
        t.group = 0; t.row0 = tm * BM; t.row_end = min(g.m, t.row0 + BM);
    }
    return true;
}

// One row's four consecutive columns col..col+3 of the accumulator tile.
template <typename ET>
__device__ __forceinline__ void gemm_store4(const GemmArgs& g, int row, int col, float (&v)[4], bool vec) {
    ET* y = static_cast<ET*>(g.y);
    if (g.bias) {
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] += g.bias[min(col + e, g.n - 1)];
    }
    if (vec) {
        if (col >= g.n) return;
        if (col >= g.n_split) {
            *reinterpret_cast<float4*>(g.y32 + (size_t)row * g.ldy32 + (col - g.n_split)) = make_float4(v[0], v[1], v[2], v[3]);
        } else if (g.glu) {
            ET* d = y + (size_t)row * g.ldy + (col >> 1);
            d[0] = (ET)glu_f(g.glu, v[0], v[1], g.limit);
            d[1] = (ET)glu_f(g.glu, v[2], v[3], g.limit);
        } else if constexpr (std::is_same<ET, float>::value) {
            *reinterpret_cast<float4*>(y + (size_t)row * g.ldy + col) = make_float4(v[0], v[1], v[2], v[3]);
        } else {
            bf16x4 o;
#pragma unroll
            for (int e = 0; e < 4; e++) o[e] = (bf16_t)v[e];
            *reinterpret_cast<bf16x4*>(y + (size_t)row * g.ldy + col) = o;
        }
        return;
    }
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int c = col + e;
        if (c >= g.n) return;
        if (c >= g.n_split) g.y32[(size_t)row * g.ldy32 + (c - g.n_split)] = v[e];
        else if (!g.glu) y[(size_t)row * g.ldy + c] = (ET)v[e];
        else if ((c & 1) == 0) y[(size_t)row * g.ldy + (c >> 1)] = (ET)glu_f(g.glu, v[e], v[(e + 1) & 3], g.limit);
    }
}

// The accumulator tile of a wave turns through a private LDS patch so that a lane owns four consecutive columns.
template <typename ET, int TM, int TN>
__device__ __forceinline__ void gemm_epilogue(const GemmArgs& g, const GemmTile& t, int col0, int wm, int wn, int lane, float* patch,
                                              f32x16 (&acc)[TM][TN]) {
    constexpr int EP = 36;
    const int pr = lane >> 3, pc = (lane & 7) * 4;
    // four columns never straddle the split, and every store address is a multiple of the store's size
    const bool vec = (g.n & 3) == 0 && (g.n_split & 3) == 0 && (g.ldy & 3) == 0 && (g.ldy32 & 3) == 0;
#pragma unroll
    for (int j = 0; j < TN; j++)
#pragma unroll
        for (int i = 0; i < TM; i++) {
#pragma unroll
            for (int r = 0; r < 16; r++) patch[((r >> 2) * 8 + (lane >> 5) * 4 + (r & 3)) * EP + (lane & 31)] = acc[i][j][r];
            __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
            __builtin_amdgcn_wave_barrier();
            __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
            for (int p = 0; p < 4; p++) {
                const int lr = p * 8 + pr, row = t.row0 + wm + i * 32 + lr;
                const f32x4 q = *reinterpret_cast<const f32x4*>(patch + lr * EP + pc);
                float v[4] = {q[0], q[1], q[2], q[3]};
                if (row < t.row_end) gemm_store4<ET>(g, row, col0 + wn + j * 32 + pc, v, vec);
            }
            __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
            __builtin_amdgcn_wave_barrier();
            __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        }
}

template <int BM, int BN, int STAGES, int WPE, int NW>
__global__ __launch_bounds__(NW * 64, WPE) void gemm_bf16_dma_kernel(GemmArgs g, int tiles_m, int tiles_n) {
    constexpr int BKB = 128, GW = NW, WGN = GW / 2;
    constexpr int WM = BM / 2, WN = BN / WGN, TM = WM / 32, TN = WN / 32;
    constexpr int CPR = BKB / 16, RPI = 64 / CPR;
    constexpr int A_INSTR = BM / (GW * RPI), B_INSTR = BN / (GW * RPI);
    static_assert(A_INSTR >= 1 && B_INSTR >= 1 && TM >= 1 && TN >= 1, "tile too small for this wave count");
    constexpr int STAGE = (BM + BN) * BKB, KS = BKB / 32;
    auto rot = [](int r) { return (r >> 1) & 7; };
    extern __shared__ __attribute__((aligned(16))) int8_t gemm_smem[];

    GemmTile tl;
    int col0;
    if (!gemm_pick_tile<BM, BN>(g, tiles_m, tiles_n, tl, col0)) return;
    const int t = threadIdx.x, lane = t & 63;
    const int wave = __builtin_amdgcn_readfirstlane(t >> 6);
    const int wm = (wave / WGN) * WM, wn = (wave % WGN) * WN;
    const int8_t* const a = static_cast<const int8_t*>(g.a);
    const int8_t* const w = static_cast<const int8_t*>(g.w) + (size_t)tl.group * g.w_stride * sizeof(bf16_t);

    unsigned offa[A_INSTR], offb[B_INSTR];
#pragma unroll
    for (int j = 0; j < A_INSTR; j++) {
        const int r = (wave * A_INSTR + j) * RPI + lane / CPR;
        int row = min(tl.row0 + r, tl.row_end - 1);
        if (g.row_src) row = g.row_src[row];
        offa[j] = (unsigned)row * (unsigned)g.lda * 2u + (unsigned)(((lane % CPR) ^ rot(r)) * 16);
    }
#pragma unroll
    for (int j = 0; j < B_INSTR; j++) {
        const int r = (wave * B_INSTR + j) * RPI + lane / CPR;
        offb[j] = (unsigned)min(col0 + r, g.n - 1) * (unsigned)g.ldw * 2u + (unsigned)(((lane % CPR) ^ rot(r)) * 16);
    }
    const unsigned lds0 = (unsigned)(uintptr_t)(__attribute__((address_space(3))) void*)gemm_smem;
    auto issue_stage = [&](int kt) {
        const unsigned sb = lds0 + (unsigned)(kt % STAGES) * STAGE;
        const size_t koff = (size_t)kt * BKB;
#pragma unroll
        for (int j = 0; j < A_INSTR; j++) gemm_dma_issue(a + koff, offa[j], sb + (wave * A_INSTR + j) * 1024);
#pragma unroll
        for (int j = 0; j < B_INSTR; j++) gemm_dma_issue(w + koff, offb[j], sb + BM * BKB + (wave * B_INSTR + j) * 1024);
    };

    f32x16 acc[TM][TN];
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) acc[i][j][r] = 0.0f;

    const int nk = g.k * 2 / BKB;
    constexpr int PER = A_INSTR + B_INSTR;
    // everything the compiler loaded itself (tile table, gathered row numbers) has to be in before the counted loads start
    gemm_wait_vmcnt<0>();
#pragma unroll
    for (int s0 = 0; s0 < STAGES - 1; s0++)
        if (s0 < nk) issue_stage(s0);
    const int fr = lane & 31, fg = lane >> 5;
    auto read_frags = [&](int kt, int ks, bf16x8 (&fa)[TM], bf16x8 (&fb)[TN]) {
        const int8_t* sa = gemm_smem + (kt % STAGES) * STAGE;
        const int8_t* sb = sa + BM * BKB;
#pragma unroll
        for (int i = 0; i < TM; i++) {
            const int r = wm + i * 32 + fr;
            fa[i] = *reinterpret_cast<const bf16x8*>(sa + r * BKB + (((ks * 2 + fg) ^ rot(r)) * 16));
        }
#pragma unroll
        for (int j = 0; j < TN; j++) {
            const int r = wn + j * 32 + fr;
            fb[j] = *reinterpret_cast<const bf16x8*>(sb + r * BKB + (((ks * 2 + fg) ^ rot(r)) * 16));
        }
    };
    auto mma = [&](const bf16x8 (&fa)[TM], const bf16x8 (&fb)[TN]) {
#pragma unroll
        for (int i = 0; i < TM; i++)
#pragma unroll
            for (int j = 0; j < TN; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
    };
    auto wait_stage = [&](int kt) {
        const int younger = min(STAGES - 2, nk - 1 - kt);
        if (younger >= 2) gemm_wait_vmcnt<2 * PER>();
        else if (younger == 1) gemm_wait_vmcnt<PER>();
        else gemm_wait_vmcnt<0>();
    };
    static_assert(STAGES <= 4 && 2 * PER < 64, "the wait distinguishes up to two younger stages");

    bf16x8 fa0[TM], fb0[TN], fa1[TM], fb1[TN];
    wait_stage(0);
    __syncthreads();
    read_frags(0, 0, fa0, fb0);
    for (int kt = 0; kt < nk; kt++) {
#pragma unroll
        for (int ks = 0; ks < KS; ks += 2) {
            read_frags(kt, ks + 1, fa1, fb1);
            if (ks == 0 && kt + STAGES - 1 < nk) issue_stage(kt + STAGES - 1);
            __builtin_amdgcn_sched_barrier(0);
            mma(fa0, fb0);
            __builtin_amdgcn_sched_barrier(0);
            if (ks + 2 < KS) {
                read_frags(kt, ks + 2, fa0, fb0);
            } else if (kt + 1 < nk) {
                wait_stage(kt + 1);
                __syncthreads();
                read_frags(kt + 1, 0, fa0, fb0);
            }
            __builtin_amdgcn_sched_barrier(0);
            mma(fa1, fb1);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    __syncthreads();
    gemm_epilogue<bf16_t, TM, TN>(g, tl, col0, wm, wn, lane, reinterpret_cast<float*>(gemm_smem) + wave * (32 * 36), acc);
}

constexpr int gemm_bf16_lds(int bm, int bn, int stages, int nw) {
    const int ring = stages * (bm + bn) * 128, epi = nw * 32 * 36 * 4;
    return ring > epi ? ring : epi;
}

template <int BM, int BN, int STAGES, int WPE, int NW>
static int launch_bf16(const GemmArgs& g, hipStream_t st) {
    constexpr int lds = gemm_bf16_lds(BM, BN, STAGES, NW);
    static std::atomic<bool> opted_in{false};
    if (!opted_in.load(std::memory_order_acquire)) {
        FX_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(gemm_bf16_dma_kernel<BM, BN, STAGES, WPE, NW>),
                                   hipFuncAttributeMaxDynamicSharedMemorySize, lds));
        opted_in.store(true, std::memory_order_release);
    }
    const int tm = g.tiles ? g.max_tiles : (g.m + BM - 1) / BM, tn = (g.n + BN - 1) / BN;
    gemm_bf16_dma_kernel<BM, BN, STAGES, WPE, NW><<<tm * tn, NW * 64, lds, st>>>(g, tm, tn);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

// A few float32 output columns (router rows, low-rank gate inputs): 16 rows x 16 columns per workgroup on
// v_mfma_f32_16x16x32_bf16, the four waves sharing k; operands straight from memory, eight k-steps in flight.
__global__ __launch_bounds__(256) void gemm_bf16_narrow_kernel(GemmArgs g, int n0) {
    __shared__ float part[4][16 * 17];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, row0 = blockIdx.x * 16, col0 = n0 + blockIdx.y * 16;
    const int r = min(row0 + (lane & 15), g.m - 1), c = min(col0 + (lane & 15), g.n - 1), kq = (lane >> 4) * 8;
    const bf16_t* a = static_cast<const bf16_t*>(g.a) + (size_t)r * g.lda + kq;
    const bf16_t* w = static_cast<const bf16_t*>(g.w) + (size_t)c * g.ldw + kq;
    f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
    constexpr int B = 8;
    for (int k0 = wave * 32 * B; k0 < g.k; k0 += 4 * 32 * B) {
        bf16x8 fa[B], fb[B];
#pragma unroll
        for (int i = 0; i < B; i++) {
            const int k = min(k0 + i * 32, g.k - 32);     // k is a multiple of 64; steps beyond it are left out below
            fa[i] = *reinterpret_cast<const bf16x8*>(a + k);
            fb[i] = *reinterpret_cast<const bf16x8*>(w + k);
        }
#pragma unroll
        for (int i = 0; i < B; i++)
            if (k0 + i * 32 < g.k) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[i], fb[i], acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) part[wave][((lane >> 4) * 4 + i) * 17 + (lane & 15)] = acc[i];
    __syncthreads();
    const int rr = t >> 4, cc = t & 15;
    const float v = (part[0][rr * 17 + cc] + part[1][rr * 17 + cc]) + (part[2][rr * 17 + cc] + part[3][rr * 17 + cc]);
    if (row0 + rr < g.m && col0 + cc < g.n) g.y32[(size_t)(row0 + rr) * g.ldy32 + (col0 + cc - g.n_split)] = g.bias ? v + g.bias[col0 + cc] : v;
}

int gemm_group_tile_rows(int rows_per_group) { return rows_per_group >= 96 ? 128 : 64; }

static int gemm_check(GemmArgs& g, size_t a_rows, int es) {
    if (!g.ldw) g.ldw = g.k;
    FX_REQUIRE(g.a && g.w && g.m > 0 && g.n > 0 && g.k > 0 && g.k % kKPad == 0 && g.lda >= g.k && g.lda % 8 == 0 && g.ldw >= g.k && g.ldw % 8 == 0,
               "gemm_float: m=%d n=%d k=%d lda=%d", g.m, g.n, g.k, g.lda);
    FX_REQUIRE((size_t)a_rows * g.lda * es < (1ull << 31) && (size_t)g.n * g.ldw * es < (1ull << 31), "gemm_float: operands beyond 2 GiB");
    FX_REQUIRE(g.n_split >= 0 && g.n_split <= g.n && (g.n_split == 0 || g.y) && (g.n_split == g.n || g.y32), "gemm_float: output pointers");
    FX_REQUIRE(!g.glu || g.n_split % 2 == 0, "gemm_float: odd number of gate/up rows");
    FX_REQUIRE(!g.tiles || (g.n_tiles && g.max_tiles > 0), "gemm_float: tile table");
    return FLEXLLM_OK;
}

template <>
int gemm_float<bf16_t>(const GemmArgs& args, hipStream_t st) {
    GemmArgs g = args;
    int rc = gemm_check(g, g.m, 2);
    if (rc) return rc;
    FX_REQUIRE(!g.tiles, "gemm_float: a tile table goes to gemm_grouped");
    // a few float32 columns behind whole tiles would cost a tile column of their own: they get the narrow kernel
    const int extra = g.n - g.n_split;
    if (g.n_split > 0 && extra > 0 && extra <= 256 && (g.n + 127) / 128 > (g.n_split + 127) / 128) {
        gemm_bf16_narrow_kernel<<<dim3((g.m + 15) / 16, (extra + 15) / 16), 256, 0, st>>>(g, g.n_split);
        FX_LAUNCH_CHECK();
        g.n = g.n_split;
    }
    auto tiles = [&](int bm, int bn) { return ((g.m + bm - 1) / bm) * ((g.n + bn - 1) / bn); };
    const int t256 = tiles(256, 256);
    if (t256 >= 256 && (t256 % 256 == 0 || t256 >= 1024)) return launch_bf16<256, 256, 2, 2, 8>(g, st);
    if (tiles(128, 128) >= 256) return launch_bf16<128, 128, 2, 2, 4>(g, st);
    if (tiles(64, 64) >= 768) return launch_bf16<64, 64, 3, 3, 4>(g, st);
    return launch_bf16<64, 64, 4, 2, 4>(g, st);
}

template <int BM>
static int gemm_grouped_bf16(const GemmArgs& args, hipStream_t st) {
    GemmArgs g = args;
    int rc = gemm_check(g, g.m, 2);
    if (rc) return rc;
    if constexpr (BM == 128) return launch_bf16<128, 128, 2, 2, 4>(g, st);
    else return launch_bf16<64, 64, 3, 3, 4>(g, st);
}

// ---- float32 -----------------------------------------------------------------------------------------------------
// 64x64 tile, four waves 2x2, 16 k per step staged through registers.
template <int BM>
__global__ __launch_bounds__(256) void gemm_f32_kernel(GemmArgs g, int tiles_m, int tiles_n) {
    constexpr int BN = 64, BK = 16, P = 65, TM = BM / 64;
    __shared__ float la[BK][BM + 1], lb[BK][P];
    __shared__ float patch[4][32 * 36];
    GemmTile tl;
    int col0;
    if (!gemm_pick_tile<BM, BN>(g, tiles_m, tiles_n, tl, col0)) return;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int wm = (wave >> 1) * (BM / 2), wn = (wave & 1) * 32;
    const float* a = static_cast<const float*>(g.a);
    const float* w = static_cast<const float*>(g.w) + (size_t)tl.group * g.w_stride;
    f32x16 acc[TM][1];
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) acc[i][0][r] = 0.0f;
    for (int k0 = 0; k0 < g.k; k0 += BK) {
        __syncthreads();
        for (int c = t; c < BM * 4; c += 256) {
            int row = min(tl.row0 + (c >> 2), tl.row_end - 1);
            if (g.row_src) row = g.row_src[row];
            const float4 v = *reinterpret_cast<const float4*>(a + (size_t)row * g.lda + k0 + (c & 3) * 4);
            la[(c & 3) * 4][c >> 2] = v.x; la[(c & 3) * 4 + 1][c >> 2] = v.y; la[(c & 3) * 4 + 2][c >> 2] = v.z; la[(c & 3) * 4 + 3][c >> 2] = v.w;
        }
        {
            const int c = t;
            const float4 v = *reinterpret_cast<const float4*>(w + (size_t)min(col0 + (c >> 2), g.n - 1) * g.ldw + k0 + (c & 3) * 4);
            lb[(c & 3) * 4][c >> 2] = v.x; lb[(c & 3) * 4 + 1][c >> 2] = v.y; lb[(c & 3) * 4 + 2][c >> 2] = v.z; lb[(c & 3) * 4 + 3][c >> 2] = v.w;
        }
        __syncthreads();
#pragma unroll
        for (int s = 0; s < BK / 2; s++) {
            const float fb = lb[2 * s + (lane >> 5)][wn + (lane & 31)];
#pragma unroll
            for (int i = 0; i < TM; i++) {
                const float fa = la[2 * s + (lane >> 5)][wm + i * 32 + (lane & 31)];
                acc[i][0] = __builtin_amdgcn_mfma_f32_32x32x2f32(fa, fb, acc[i][0], 0, 0, 0);
            }
        }
    }
    gemm_epilogue<float, TM, 1>(g, tl, col0, wm, wn, lane, patch[wave], acc);
}

template <int BM>
static int launch_f32(const GemmArgs& args, hipStream_t st) {
    GemmArgs g = args;
    int rc = gemm_check(g, g.m, 4);
    if (rc) return rc;
    const int tm = g.tiles ? g.max_tiles : (g.m + BM - 1) / BM, tn = (g.n + 63) / 64;
    gemm_f32_kernel<BM><<<tm * tn, 256, 0, st>>>(g, tm, tn);
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

template <>
int gemm_float<float>(const GemmArgs& g, hipStream_t st) { return launch_f32<64>(g, st); }

template <typename ET>
int gemm_grouped(const GemmArgs& g, int tile_rows, hipStream_t st) {
    FX_REQUIRE(g.tiles && (tile_rows == 64 || tile_rows == 128), "gemm_grouped: tile table of %d rows", tile_rows);
    if constexpr (std::is_same<ET, float>::value) return tile_rows == 128 ? launch_f32<128>(g, st) : launch_f32<64>(g, st);
    else return tile_rows == 128 ? gemm_grouped_bf16<128>(g, st) : gemm_grouped_bf16<64>(g, st);
}
template int gemm_grouped<bf16_t>(const GemmArgs&, int, hipStream_t);
template int gemm_grouped<float>(const GemmArgs&, int, hipStream_t);

}  // namespace fx

using namespace fx;

extern "C" {

int flexllm_linear_float_gemm(const void* a, const void* w, const float* bias, void* y, float* y32, int m, int k, int n, int n_split, int glu, float limit,
                              int dtype, void* stream) {
    FX_REQUIRE((dtype == 0 || dtype == 1) && glu >= 0 && glu <= 1 + FLEXLLM_GLU_GELU, "linear_float_gemm: dtype=%d glu=%d", dtype, glu);
    GemmArgs g;
    g.a = a; g.w = w; g.lda = k; g.m = m; g.n = n; g.k = k; g.n_split = n_split; g.glu = glu; g.limit = limit; g.bias = bias;
    g.y = y; g.ldy = glu ? n_split / 2 : n_split; g.y32 = y32; g.ldy32 = n - n_split;
    return dtype == 0 ? gemm_float<bf16_t>(g, as_stream(stream)) : gemm_float<float>(g, as_stream(stream));
}

}  // extern "C"
