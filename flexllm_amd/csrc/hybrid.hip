// Decoder of floating-point layers (latent attention, attention over shared key/value rows, gated linear attention, dense or
// mixture feed-forwards) on one GPU: owns the repacked weights, the slots with the sequences' cached rows and states, and
// the workspace, and strings the kernels of float_ops.h together.
//
// A layer run is one pass through a layer: layers inside the loop have several, with the same weights and rows or states of
// their own.
//
// Two schedules over the same weights and slots: up to kSmallTokens tokens go through the one-token linears with float32
// activations (decode: every quantity that changes between steps is read from the slot's device state, so one captured
// graph serves every token), more go through the GEMMs in pieces of at most kPieceTokens.  In both, the norm after a
// sublayer, the residual and the norm before the next one are one step: the sublayer's output is kept "pending" until the
// next sublayer's first kernel takes it in.
#include "float_ops.h"
#include "logits_kernels.h"
#include <math.h>
#include <string.h>
#include <vector>

namespace fx {

constexpr int kSmallTokens = 8;
constexpr int kPieceTokens = 4096;
constexpr int kHeadRows = 256;          // rows of logits formed at a time
constexpr int kAbsorbTokens = 16;       // tokens per launch of the attention kernels for few tokens

static inline int up4(int v) { return (v + 3) / 4 * 4; }

struct HybridLayer {
    flexllm_hybrid_layer d;
    float *g1 = nullptr, *g1b = nullptr, *g2 = nullptr, *g2b = nullptr;       // effective norm weights
    void *w_in = nullptr, *w_o = nullptr;     // latent: [q; dkv]; shared key/value: [q; k]; gated linear: [q; k; v; g; a1]
    float* in_bias = nullptr;                 // [n_in]
    int n_in = 0, n_et = 0, k_o = 0;          // rows of w_in, those that stay in ET, width of w_o's input
    void *uk = nullptr, *uv = nullptr;
    float* latent_norm = nullptr;
    float *cos_t = nullptr, *sin_t = nullptr;
    void* a2 = nullptr;
    float *a2_bias = nullptr, *head_norm = nullptr;
    void *w_gu = nullptr, *w_d = nullptr;     // dense, or the experts one after the other
    void *w_side = nullptr, *w_sd = nullptr;  // mixture: [shared gate/up; router; shared gate row], shared down
    int n_side = 0;
    float* kv_norm = nullptr;                 // product of the query and key norms' weights
    LatentDims ld = {};
    SharedKvDims sd = {};
    GlaDims gd = {};
};

struct LayerRun { int layer; bool again; };        // again: the embedding output is added ahead of it

struct HybridSlot {
    // per layer run
    std::vector<void*> rows;                  // cached rows (own or, with kv_from, the other layer's)
    std::vector<float*> inv_rms;              // shared key/value: what the rows' products are multiplied by
    std::vector<float*> state;                // gated linear attention state
    int* pos = nullptr;                       // device: [0] tokens held, [1] step of the decode loop, [3] error flag
    int length = 0;
};

}  // namespace fx

struct flexllm_hybrid {
    flexllm_hybrid_config cfg;
    std::vector<fx::HybridLayer> layers;
    std::vector<fx::LayerRun> runs;
    std::vector<fx::HybridSlot> slots;
    std::vector<void*> owned, pool;           // pool: the many-token workspace
    uint16_t* embed = nullptr;
    void* head = nullptr;
    float* g_final = nullptr;
    // largest sizes over the layers
    int max_et = 0, max_f32 = 0, max_att = 0, max_ff = 0, max_slots_ff = 1, max_shared = 0, max_route = 4, max_experts = 0, max_top = 1;
    size_t absorbed = 0;                      // scratch floats per token of the attention kernels for few tokens
    // one-token workspace
    float *x0 = nullptr, *xa = nullptr, *xb = nullptr, *proj = nullptr, *f32 = nullptr, *att = nullptr, *y = nullptr, *hn = nullptr, *hid = nullptr, *hs = nullptr, *route = nullptr;
    float *pick_w = nullptr, *scratch = nullptr, *logits = nullptr, *hw = nullptr;
    int *pick = nullptr, *want = nullptr;
    float* am_v = nullptr;
    int* am_i = nullptr;
    float* topk_val = nullptr;
    int* topk_idx = nullptr;
    int* gen_token = nullptr;
    // many-token workspace
    int rows = 0;
    float *lx0 = nullptr, *lx = nullptr, *lf32 = nullptr, *ly = nullptr, *lys = nullptr, *lroute = nullptr, *lgla = nullptr, *lpick_w = nullptr;
    void *lh = nullptr, *lproj = nullptr, *latt = nullptr, *lhid = nullptr, *lhs = nullptr, *lk = nullptr, *lvt = nullptr, *lhead = nullptr;
    int *lpick = nullptr, *lpos_of = nullptr, *lrow_src = nullptr, *lcounts = nullptr, *lntiles = nullptr;
    int4* ltiles = nullptr;
    // captured decode step
    hipGraphExec_t graph = nullptr;
    int graph_slot = -1, graph_topk = 0;
    const void *graph_io = nullptr, *graph_out = nullptr, *graph_rands = nullptr;
    hipStream_t graph_stream = nullptr;
};

namespace fx {

static int halloc(std::vector<void*>& list, void** p, size_t bytes) {
    const size_t n = (bytes + 255) / 256 * 256 + 256;
    hipError_t e = hipMalloc(p, n);
    if (e != hipSuccess) {
        set_error("hipMalloc(%zu) failed: %s", n, hipGetErrorString(e));
        *p = nullptr;
        return e == hipErrorOutOfMemory ? FLEXLLM_ENOMEM : FLEXLLM_EHIP;
    }
    list.push_back(*p);
    FX_HIP(hipMemset(*p, 0, n));             // padding columns are multiplied by zero weights: they have to be finite
    return FLEXLLM_OK;
}
#define FX_TRY(expr)              \
    do {                          \
        int rc_ = (expr);         \
        if (rc_) return rc_;      \
    } while (0)

static inline const bf16_t* as_bf16(const uint16_t* p) { return reinterpret_cast<const bf16_t*>(p); }

// ---- creation ------------------------------------------------------------------------------------------------------
template <typename T>
static int own(flexllm_hybrid* m, T*& p, size_t count) { return halloc(m->owned, reinterpret_cast<void**>(&p), count * sizeof(T)); }

static int own_norm(flexllm_hybrid* m, float*& dst, const uint16_t* src, int n, float add, const char* what) {
    FX_REQUIRE(src, "hybrid_create: missing tensor %s", what);
    FX_TRY(own(m, dst, n));
    return widen_rows(as_bf16(src), dst, n, add, nullptr);
}

// A matrix of `rows` rows in ET with padded row length, filled piece by piece.
template <typename ET>
struct Packer {
    flexllm_hybrid* m;
    ET* dst = nullptr;
    int k, kpad, next = 0;
    Packer(flexllm_hybrid* m_, int k_) : m(m_), k(k_), kpad(pad_k(k_)) {}
    int alloc(size_t rows) { return halloc(m->owned, reinterpret_cast<void**>(&dst), rows * kpad * sizeof(ET)); }
    int put(const uint16_t* src, int n, const char* what, int step = 1, int off = 0) {
        FX_REQUIRE(src, "hybrid_create: missing tensor %s", what);
        FX_TRY(pack_rows<ET>(as_bf16(src), dst + (size_t)next * kpad, n, k, kpad, step, off, nullptr));
        if (step == 1) next += n;
        return FLEXLLM_OK;
    }
    // rows of heads that lie `padded` rows apart
    int put_heads(const uint16_t* src, int heads, int dim, int padded, const char* what) {
        for (int h = 0; h < heads; h++) {
            FX_TRY(put(src ? src + (size_t)h * dim * k : nullptr, dim, what));
            next += padded - dim;
        }
        return FLEXLLM_OK;
    }
    int put_pair(const uint16_t* gate, const uint16_t* up, int n, const char* what) {
        FX_TRY(put(gate, n, what, 2, 0));
        FX_TRY(put(up, n, what, 2, 1));
        next += 2 * n;
        return FLEXLLM_OK;
    }
};

static int host_floats(const uint16_t* src, int n, std::vector<float>& out) {
    std::vector<uint16_t> u(n);
    FX_HIP(hipMemcpy(u.data(), src, n * sizeof(uint16_t), hipMemcpyDeviceToHost));
    out.resize(n);
    for (int i = 0; i < n; i++) {
        const uint32_t w = (uint32_t)u[i] << 16;
        memcpy(&out[i], &w, 4);
    }
    return FLEXLLM_OK;
}
static int own_floats(flexllm_hybrid* m, float*& dst, const std::vector<float>& v) {
    FX_TRY(own(m, dst, v.size()));
    FX_HIP(hipMemcpy(dst, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
    return FLEXLLM_OK;
}

// Rotation tables: neighbouring pairs; with yarn the frequencies of slow pairs are divided by the factor, with a ramp
// between the pairs that turn `fast` and `slow` times over the original length, and sine and cosine are scaled.
static int rotation_tables(flexllm_hybrid* m, const flexllm_hybrid_layer& d, float*& cos_t, float*& sin_t) {
    const int half = d.rot_dim / 2, P = m->cfg.max_pos;
    std::vector<float> c((size_t)P * half), s((size_t)P * half);
    std::vector<double> f(half);
    double mag = 1.0, lo = 0.0, hi = 0.0;
    if (d.yarn) {
        auto turns = [&](double t) { return d.rot_dim * log(d.yarn_original / (2.0 * M_PI * t)) / (2.0 * log(d.rot_base)); };
        lo = fmax(floor(turns(d.yarn_fast)), 0.0);
        hi = fmin(ceil(turns(d.yarn_slow)), d.rot_dim - 1.0);
        mag = 0.1 * log(d.yarn_factor) + 1.0;
    }
    for (int i = 0; i < half; i++) {
        f[i] = pow(d.rot_base, -2.0 * i / d.rot_dim);
        if (d.yarn) {
            const double ramp = fmin(fmax((i - lo) / fmax(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / d.yarn_factor * ramp + f[i] * (1.0 - ramp);
        }
    }
    for (int p = 0; p < P; p++)
        for (int i = 0; i < half; i++) {
            c[(size_t)p * half + i] = (float)(mag * cos(p * f[i]));
            s[(size_t)p * half + i] = (float)(mag * sin(p * f[i]));
        }
    FX_TRY(own(m, cos_t, c.size()));
    FX_TRY(own(m, sin_t, s.size()));
    FX_HIP(hipMemcpy(cos_t, c.data(), c.size() * sizeof(float), hipMemcpyHostToDevice));
    FX_HIP(hipMemcpy(sin_t, s.data(), s.size() * sizeof(float), hipMemcpyHostToDevice));
    return FLEXLLM_OK;
}

static int check_layer(const flexllm_hybrid_config& c, const flexllm_hybrid_layer* all, int i) {
    const flexllm_hybrid_layer& d = all[i];
    FX_REQUIRE(d.heads > 0 && d.dim > 0 && d.vdim > 0, "hybrid_create: layer %d: heads=%d dim=%d vdim=%d", i, d.heads, d.dim, d.vdim);
    if (d.mixer == FLEXLLM_MIX_LATENT) {
        FX_REQUIRE(d.rot_dim > 0 && d.rot_dim % 2 == 0 && d.kv_rank > 0 && d.window >= 0 && d.rot_base > 0.0, "hybrid_create: layer %d: rot_dim=%d kv_rank=%d window=%d", i, d.rot_dim, d.kv_rank, d.window);
        FX_REQUIRE(d.kv_from < i, "hybrid_create: layer %d reads the rows of layer %d", i, d.kv_from);
        if (d.kv_from >= 0) {
            const flexllm_hybrid_layer& s = all[d.kv_from];
            FX_REQUIRE(s.mixer == FLEXLLM_MIX_LATENT && s.kv_from < 0 && s.kv_rank == d.kv_rank && s.rot_dim == d.rot_dim,
                       "hybrid_create: layer %d cannot read the rows of layer %d", i, d.kv_from);
        }
    } else if (d.mixer == FLEXLLM_MIX_SHARED_KV) {
        FX_REQUIRE(d.kv_heads > 0 && d.heads % d.kv_heads == 0 && d.vdim == d.dim && d.dim <= 512, "hybrid_create: layer %d: %d heads on %d, dim=%d vdim=%d (at most 512)",
                   i, d.heads, d.kv_heads, d.dim, d.vdim);
        FX_REQUIRE(d.temp_coef == 0.0f || d.temp_every > 0, "hybrid_create: layer %d: temp_every=%d", i, d.temp_every);
    } else {
        FX_REQUIRE(d.mixer == FLEXLLM_MIX_GLA && d.a_rank > 0 && d.tau > 0.0f, "hybrid_create: layer %d: mixer=%d a_rank=%d tau=%g", i, d.mixer, d.a_rank, (double)d.tau);
    }
    FX_REQUIRE(d.ff_kind >= FLEXLLM_FF_NONE && d.ff_kind <= FLEXLLM_FF_MOE, "hybrid_create: layer %d: ff_kind=%d", i, d.ff_kind);
    FX_REQUIRE(d.glu == FLEXLLM_GLU_CLAMPED || d.glu == FLEXLLM_GLU_GELU, "hybrid_create: layer %d: glu=%d", i, d.glu);
    FX_REQUIRE(d.ff_kind == FLEXLLM_FF_NONE || d.ff > 0, "hybrid_create: layer %d: ff=%d", i, d.ff);
    FX_REQUIRE(d.ff_kind != FLEXLLM_FF_MOE || (d.experts > 0 && d.experts <= 1024 && d.top > 0 && d.top <= 32 && d.top <= d.experts && d.shared_ff >= 0),
               "hybrid_create: layer %d: %d experts, top %d", i, d.experts, d.top);
    const int longest = c.width > d.heads * d.vdim ? c.width : d.heads * d.vdim;
    FX_REQUIRE(pad_k(longest) <= 15360 && pad_k(d.ff) <= 15360, "hybrid_create: layer %d: a vector of %d or %d exceeds LDS", i, longest, d.ff);
    return FLEXLLM_OK;
}

template <typename ET>
static int create_layer(flexllm_hybrid* m, int i, const flexllm_hybrid_layer_weights& w) {
    HybridLayer& L = m->layers[i];
    const flexllm_hybrid_layer& d = L.d;
    const flexllm_hybrid_config& c = m->cfg;
    const int W = c.width;
    FX_TRY(own_norm(m, L.g1, w.norm1, W, c.norm_add, "norm1"));
    if (c.post_norms) FX_TRY(own_norm(m, L.g1b, w.norm1b, W, c.norm_add, "norm1b"));
    Packer<ET> in(m, W), out(m, d.heads * d.vdim);
    if (d.mixer == FLEXLLM_MIX_LATENT) {
        const int nq = d.heads * (d.dim + d.rot_dim), nk = d.kv_from < 0 ? d.kv_rank + d.rot_dim : 0;
        L.n_et = nq;
        L.n_in = nq + up4(nk);
        FX_TRY(in.alloc(L.n_in));
        FX_TRY(in.put(w.q, nq, "mix.q"));
        if (nk) FX_TRY(in.put(w.dkv, nk, "mix.dkv"));
        LatentDims& ld = L.ld;
        ld.heads = d.heads; ld.dim = d.dim; ld.rot_dim = d.rot_dim; ld.vdim = d.vdim; ld.kv_rank = d.kv_rank;
        ld.kvp = pad_k(d.kv_rank); ld.ldc = ld.kvp + (d.rot_dim + 7) / 8 * 8;
        ld.window = d.window; ld.scale = d.scale; ld.eps = c.eps; ld.capacity = c.max_pos;
        Packer<ET> uk(m, d.kv_rank), uv(m, d.kv_rank);
        FX_TRY(uk.alloc((size_t)d.heads * d.dim));
        FX_TRY(uk.put(w.uk, d.heads * d.dim, "mix.uk"));
        FX_TRY(uv.alloc((size_t)d.heads * d.vdim));
        FX_TRY(uv.put(w.uv, d.heads * d.vdim, "mix.uv"));
        L.uk = uk.dst; L.uv = uv.dst;
        if (nk) FX_TRY(own_norm(m, L.latent_norm, w.dkv_norm, d.kv_rank, 0.0f, "mix.dkv.norm"));
        for (int j = 0; j < i && !L.cos_t; j++) {         // one table per distinct rotation
            const flexllm_hybrid_layer& o = m->layers[j].d;
            if (o.mixer == FLEXLLM_MIX_LATENT && o.rot_dim == d.rot_dim && o.rot_base == d.rot_base && o.yarn == d.yarn && o.yarn_factor == d.yarn_factor &&
                o.yarn_original == d.yarn_original && o.yarn_fast == d.yarn_fast && o.yarn_slow == d.yarn_slow) {
                L.cos_t = m->layers[j].cos_t; L.sin_t = m->layers[j].sin_t;
            }
        }
        if (!L.cos_t) FX_TRY(rotation_tables(m, d, L.cos_t, L.sin_t));
        const size_t a = latent_absorbed_scratch(ld);
        if (a > m->absorbed) m->absorbed = a;
    } else if (d.mixer == FLEXLLM_MIX_SHARED_KV) {
        SharedKvDims& s = L.sd;
        s.heads = d.heads; s.kv_heads = d.kv_heads; s.dim = d.dim; s.dimp = pad8(d.dim); s.sink = d.sink; s.scale = d.scale;
        s.temp_coef = d.temp_coef; s.temp_every = d.temp_every; s.eps = c.eps; s.capacity = c.max_pos;
        L.n_et = d.heads * s.dimp;
        L.n_in = L.n_et + d.kv_heads * s.dimp;
        FX_TRY(in.alloc(L.n_in));
        FX_TRY(in.put_heads(w.q, d.heads, d.dim, s.dimp, "mix.q"));
        FX_TRY(in.put_heads(w.k, d.kv_heads, d.dim, s.dimp, "mix.k"));
        std::vector<float> v, u;
        if (w.q_bias || w.k_bias) {
            std::vector<float> bias(L.n_in, 0.0f);
            auto spread = [&](const uint16_t* src, int heads, int at) {
                if (!src) return FLEXLLM_OK;
                FX_TRY(host_floats(src, heads * d.dim, v));
                for (int h = 0; h < heads; h++)
                    for (int e = 0; e < d.dim; e++) bias[at + h * s.dimp + e] = v[h * d.dim + e];
                return FLEXLLM_OK;
            };
            FX_TRY(spread(w.q_bias, d.heads, 0));
            FX_TRY(spread(w.k_bias, d.kv_heads, L.n_et));
            FX_TRY(own_floats(m, L.in_bias, bias));
        }
        FX_REQUIRE(w.q_norm && w.k_norm, "hybrid_create: missing tensor mix.q.norm or mix.k.norm");
        FX_TRY(host_floats(w.q_norm, d.dim, v));
        FX_TRY(host_floats(w.k_norm, d.dim, u));
        for (int e = 0; e < d.dim; e++) v[e] *= u[e];
        v.resize(s.dimp, 0.0f);
        FX_TRY(own_floats(m, L.kv_norm, v));
        const size_t a = shared_kv_scratch(s);
        if (a > m->absorbed) m->absorbed = a;
    } else {
        const int HD = d.heads * d.dim, HV = d.heads * d.vdim;
        L.n_et = 2 * HD + 2 * HV;
        L.n_in = L.n_et + up4(d.a_rank);
        FX_TRY(in.alloc(L.n_in));
        FX_TRY(in.put(w.q, HD, "mix.q"));
        FX_TRY(in.put(w.k, HD, "mix.k"));
        FX_TRY(in.put(w.v, HV, "mix.v"));
        FX_TRY(in.put(w.g, HV, "mix.g"));
        FX_TRY(in.put(w.a1, d.a_rank, "mix.a1"));
        Packer<ET> a2(m, d.a_rank);
        FX_TRY(a2.alloc(HD));
        FX_TRY(a2.put(w.a2, HD, "mix.a2"));
        L.a2 = a2.dst;
        FX_TRY(own_norm(m, L.a2_bias, w.a2_bias, HD, 0.0f, "mix.a2.b"));
        FX_TRY(own_norm(m, L.head_norm, w.head_norm, d.vdim, 0.0f, "mix.norm"));
        GlaDims& g = L.gd;
        g.heads = d.heads; g.dim = d.dim; g.vdim = d.vdim; g.a_rank = d.a_rank; g.tau = d.tau; g.eps = c.eps;
    }
    L.w_in = in.dst;
    L.k_o = d.heads * d.vdim;
    FX_TRY(out.alloc(W));
    FX_TRY(out.put(w.o, W, "mix.o"));
    L.w_o = out.dst;
    auto grow = [](int& v, int n) { if (n > v) v = n; };
    grow(m->max_et, up4(L.n_et));
    grow(m->max_f32, L.n_in - L.n_et);
    grow(m->max_att, L.k_o);
    if (d.ff_kind == FLEXLLM_FF_NONE) return FLEXLLM_OK;
    FX_TRY(own_norm(m, L.g2, w.norm2, W, c.norm_add, "norm2"));
    if (c.post_norms) FX_TRY(own_norm(m, L.g2b, w.norm2b, W, c.norm_add, "norm2b"));
    Packer<ET> gu(m, W), dn(m, d.ff);
    const int E = d.ff_kind == FLEXLLM_FF_MOE ? d.experts : 1;
    FX_TRY(gu.alloc((size_t)E * 2 * d.ff));
    FX_TRY(dn.alloc((size_t)E * W));
    for (int e = 0; e < E; e++) {
        if (d.ff_kind == FLEXLLM_FF_MOE) {
            FX_REQUIRE(w.expert_gate && w.expert_up && w.expert_down, "hybrid_create: missing expert tensors");
            FX_TRY(gu.put_pair(w.expert_gate[e], w.expert_up[e], d.ff, "mlp.e*.gate/up"));
            FX_TRY(dn.put(w.expert_down[e], W, "mlp.e*.down"));
        } else {
            FX_TRY(gu.put_pair(w.gate, w.up, d.ff, "mlp.gate/up"));
            FX_TRY(dn.put(w.down, W, "mlp.down"));
        }
    }
    L.w_gu = gu.dst; L.w_d = dn.dst;
    grow(m->max_ff, d.ff);
    if (d.ff_kind == FLEXLLM_FF_MOE) {
        Packer<ET> side(m, W), sd(m, d.shared_ff > 0 ? d.shared_ff : 1);
        L.n_side = 2 * d.shared_ff + up4(d.experts + 1);
        FX_TRY(side.alloc(L.n_side));
        if (d.shared_ff) FX_TRY(side.put_pair(w.shared_gate, w.shared_up, d.shared_ff, "mlp.shared.gate/up"));
        FX_TRY(side.put(w.router, d.experts, "mlp.router"));
        if (d.shared_ff) {
            FX_TRY(side.put(w.shared_sg, 1, "mlp.shared.sg"));
            FX_TRY(sd.alloc(W));
            FX_TRY(sd.put(w.shared_down, W, "mlp.shared.down"));
            L.w_sd = sd.dst;
        }
        L.w_side = side.dst;
        grow(m->max_shared, d.shared_ff);
        grow(m->max_route, up4(d.experts + 1));
        grow(m->max_experts, d.experts);
        grow(m->max_top, d.top);
    }
    return FLEXLLM_OK;
}

template <typename ET>
static int create_model(flexllm_hybrid* m, const flexllm_hybrid_weights& w, const flexllm_hybrid_layer_weights* lw) {
    const flexllm_hybrid_config& c = m->cfg;
    const int W = c.width;
    FX_REQUIRE(w.embed && w.head && w.final_norm, "hybrid_create: missing tensor embed, head or final.norm");
    FX_TRY(own(m, m->embed, (size_t)c.vocab * W));
    FX_HIP(hipMemcpy(m->embed, w.embed, (size_t)c.vocab * W * 2, hipMemcpyDeviceToDevice));
    FX_TRY(own_norm(m, m->g_final, w.final_norm, W, c.norm_add, "final.norm"));
    if (w.head == w.embed && std::is_same<ET, bf16_t>::value && pad_k(W) == W) {
        m->head = m->embed;                               // tied, and already in the head's layout
    } else {
        Packer<ET> head(m, W);
        FX_TRY(head.alloc(c.vocab));
        FX_TRY(head.put(w.head, c.vocab, "head"));
        m->head = head.dst;
    }
    for (int i = 0; i < c.layers; i++) FX_TRY(create_layer<ET>(m, i, lw[i]));
    m->slots.resize(c.slots);
    for (HybridSlot& s : m->slots) {
        const int n = (int)m->runs.size();
        s.rows.resize(n); s.inv_rms.resize(n); s.state.resize(n);
        FX_TRY(own(m, s.pos, 8));
        std::vector<int> latest(c.layers, -1);            // the last run of a layer so far
        for (int r = 0; r < n; r++) {
            const int i = m->runs[r].layer;
            const HybridLayer& L = m->layers[i];
            if (L.d.mixer == FLEXLLM_MIX_GLA) {
                FX_TRY(own(m, s.state[r], (size_t)L.d.heads * L.d.dim * L.d.vdim));
            } else if (L.d.mixer == FLEXLLM_MIX_SHARED_KV) {
                FX_TRY(halloc(m->owned, &s.rows[r], (size_t)L.sd.kv_heads * c.max_pos * L.sd.dimp * sizeof(ET)));
                FX_TRY(own(m, s.inv_rms[r], (size_t)L.sd.kv_heads * c.max_pos));
            } else if (L.d.kv_from >= 0) {
                s.rows[r] = s.rows[latest[L.d.kv_from]];
            } else {
                FX_TRY(halloc(m->owned, &s.rows[r], (size_t)c.max_pos * L.ld.ldc * sizeof(ET)));
            }
            latest[i] = r;
        }
    }
    const size_t T = kSmallTokens;
    FX_TRY(own(m, m->x0, T * W));
    FX_TRY(own(m, m->xa, T * W));
    FX_TRY(own(m, m->xb, T * W));
    FX_TRY(own(m, m->hn, T * W));
    FX_TRY(own(m, m->y, T * W));
    FX_TRY(own(m, m->hw, T * W));
    FX_TRY(own(m, m->proj, T * m->max_et));
    FX_TRY(own(m, m->f32, T * (m->max_f32 + 4)));
    FX_TRY(own(m, m->att, T * m->max_att));
    FX_TRY(own(m, m->hid, T * m->max_top * (m->max_ff + 1)));
    FX_TRY(own(m, m->hs, T * (m->max_shared + 1)));
    FX_TRY(own(m, m->route, T * m->max_route));
    FX_TRY(own(m, m->pick, T * m->max_top));
    FX_TRY(own(m, m->pick_w, T * m->max_top));
    FX_TRY(own(m, m->scratch, (size_t)kAbsorbTokens * m->absorbed + 1));
    FX_TRY(own(m, m->logits, c.vocab));
    FX_TRY(own(m, m->want, kPieceTokens));
    FX_TRY(own(m, m->am_v, kArgmaxParts));
    FX_TRY(own(m, m->am_i, kArgmaxParts));
    FX_TRY(own(m, m->topk_val, kTopKParts * kTopKMax));
    FX_TRY(own(m, m->topk_idx, kTopKParts * kTopKMax));
    FX_TRY(own(m, m->gen_token, 1));
    FX_HIP(hipDeviceSynchronize());
    return FLEXLLM_OK;
}

// Workspace of the many-token schedule for pieces of up to `rows` tokens.
template <typename ET>
static int many_workspace(flexllm_hybrid* m, int rows) {
    if (rows <= m->rows) return FLEXLLM_OK;
    const flexllm_hybrid_config& c = m->cfg;
    FX_HIP(hipDeviceSynchronize());
    if (m->graph) { (void)hipGraphExecDestroy(m->graph); m->graph = nullptr; }
    for (void* p : m->pool) (void)hipFree(p);
    m->pool.clear();
    m->rows = 0;
    const size_t R = (rows + 63) / 64 * 64, W = c.width;
    size_t k_el = 0, vt_el = 0, gla = 0;
    for (const HybridLayer& L : m->layers) {
        if (L.d.mixer == FLEXLLM_MIX_LATENT) {
            if (std::is_same<ET, float>::value || !latent_flash_ok(L.ld)) continue;
            size_t kv = L.d.window > 0 ? R + L.d.window : (size_t)c.max_pos;
            if (kv > (size_t)c.max_pos) kv = c.max_pos;
            kv = (kv + 127) / 64 * 64;
            if (kv * L.d.heads * L.d.dim > k_el) k_el = kv * L.d.heads * L.d.dim;
            if (kv * L.d.heads * L.d.vdim > vt_el) vt_el = kv * L.d.heads * L.d.vdim;
        } else if (L.d.mixer == FLEXLLM_MIX_GLA && gla_chunks_ok(L.gd)) {
            const size_t g = gla_chunk_scratch(L.gd, (int)R);
            if (g > gla) gla = g;
        }
    }
    auto pool = [&](auto*& p, size_t count) { return halloc(m->pool, reinterpret_cast<void**>(&p), count * sizeof(*p)); };
    auto pool_et = [&](void*& p, size_t count) { return halloc(m->pool, &p, count * sizeof(ET)); };
    const size_t top = m->max_experts ? m->max_top : 1;
    FX_TRY(pool(m->lx, R * W));
    if (c.loop_times > 1) FX_TRY(pool(m->lx0, R * W));
    FX_TRY(pool(m->lf32, R * (m->max_f32 + 4)));
    FX_TRY(pool(m->ly, R * W));
    FX_TRY(pool_et(m->lh, R * pad_k((int)W)));
    FX_TRY(pool_et(m->lproj, R * ((size_t)(m->max_et + 7) / 8 * 8)));
    FX_TRY(pool_et(m->latt, R * pad_k(m->max_att)));
    FX_TRY(pool_et(m->lhid, R * top * pad_k(m->max_ff + 1)));
    FX_TRY(pool_et(m->lhead, (size_t)kHeadRows * pad_k((int)W)));
    FX_TRY(pool_et(m->lk, k_el + 1));
    FX_TRY(pool_et(m->lvt, vt_el + 1));
    FX_TRY(pool(m->lgla, gla + 1));
    if (m->max_experts) {
        FX_TRY(pool(m->lys, R * top * W));
        FX_TRY(pool_et(m->lhs, R * pad_k(m->max_shared + 1)));
        FX_TRY(pool(m->lroute, R * m->max_route));
        FX_TRY(pool(m->lpick, R * top));
        FX_TRY(pool(m->lpick_w, R * top));
        FX_TRY(pool(m->lpos_of, R * top));
        FX_TRY(pool(m->lrow_src, R * top));
        FX_TRY(pool(m->lcounts, 2 * (size_t)m->max_experts));
        FX_TRY(pool(m->lntiles, 1));
        FX_TRY(pool(m->ltiles, R * top / 64 + m->max_experts + 1));
    }
    m->rows = (int)R;
    return FLEXLLM_OK;
}

// ---- one to kSmallTokens tokens --------------------------------------------------------------------------------------
struct Pending { bool on = false; const float* gb = nullptr; };      // the last sublayer's output in y still has to be added

template <typename ET>
static int run_small(flexllm_hybrid* m, HybridSlot& s, const int* tokens, int T, const int* want, int n_want, float* logits, float* layers_out, hipStream_t st) {
    const flexllm_hybrid_config& c = m->cfg;
    const int W = c.width, kw = pad_k(W);
    float *x = m->x0, *other = m->xa;                     // the embedding output stays in x0, later residuals alternate
    Pending pend;
    FX_TRY(embed_rows_bf16(as_bf16(m->embed), c.embed_scale, tokens, T, x, W, c.vocab, &s.pos[3], st));
    auto moved = [&] {                                    // the residual now is where `other` was
        x = other;
        other = x == m->xa ? m->xb : m->xa;
        pend = Pending();
    };
    auto settle = [&] {                                   // take the pending output in, without a norm behind it
        if (!pend.on) return FLEXLLM_OK;
        RowArgs r;
        r.x = x; r.x_new = other; r.y = m->y; r.ldy = W; r.gb = pend.gb; r.eps = c.eps; r.width = W; r.rows = T;
        const int rc = norm_rows<ET>(r, st);
        moved();
        return rc;
    };
    auto pending = [&](const float* gb) { pend.on = true; pend.gb = gb; };
    auto base = [&](const void* w, int n, int k) {
        GemvArgs a;
        a.w = w; a.n = n; a.k = k; a.kpad = pad_k(k); a.eps = c.eps;
        return a;
    };
    // linear on norm(x + pending [+ x0])
    auto norm_linear = [&](GemvArgs a, const float* g, bool add_x0 = false) {
        if (add_x0 && pend.gb) FX_TRY(settle());          // the kernel takes a norm's weight or x0
        a.x = x; a.ldx = W; a.g = g;
        if (pend.on) { a.y = m->y; a.ldy = W; a.gb = pend.gb; }
        if (add_x0) a.x0 = m->x0;
        const bool changes = pend.on || add_x0;
        if (changes) a.x_new = other;
        const int rc = gemv_float<ET>(a, 1, T, st);
        if (changes) moved();
        return rc;
    };
    auto plain_linear = [&](const void* w, int n, int k, const float* v, int ldv, float* out) {
        GemvArgs a = base(w, n, k);
        a.x = v; a.ldx = ldv; a.n_split = 0; a.out32 = out; a.ldo32 = n;
        return gemv_float<ET>(a, 0, T, st);
    };
    const int runs = (int)m->runs.size();
    for (int r = 0; r < runs; r++) {
        const HybridLayer& L = m->layers[m->runs[r].layer];
        const int nf = L.n_in - L.n_et;
        if (layers_out && r > 0) {
            FX_TRY(settle());
            FX_HIP(hipMemcpyAsync(layers_out + (size_t)(r - 1) * T * W, x, sizeof(float) * T * W, hipMemcpyDeviceToDevice, st));
        }
        GemvArgs a = base(L.w_in, L.n_in, W);
        a.n_split = L.n_et; a.out = m->proj; a.ldo = m->max_et; a.out32 = m->f32; a.ldo32 = nf; a.bias = L.in_bias;
        FX_TRY(norm_linear(a, L.g1, m->runs[r].again));
        if (L.d.mixer == FLEXLLM_MIX_SHARED_KV) {
            const SharedKvRows<ET> rows = {static_cast<ET*>(s.rows[r]), s.inv_rms[r]};
            FX_TRY(shared_kv_splits<ET>(L.sd, m->proj, m->max_et, m->f32, nf, L.kv_norm, rows, s.pos, 0, T, m->scratch, m->att, m->max_att, 1, st));
        } else if (L.d.mixer == FLEXLLM_MIX_LATENT) {
            ET* rows = static_cast<ET*>(s.rows[r]);
            FX_TRY(latent_decode<ET>(L.ld, m->proj, m->max_et, nf ? m->f32 : nullptr, nf, L.latent_norm, L.cos_t, L.sin_t, static_cast<ET*>(L.uk),
                                     static_cast<ET*>(L.uv), rows, s.pos, T, m->scratch, m->att, m->max_att, st));
        } else {
            FX_TRY(gla_steps<ET>(L.gd, m->proj, m->max_et, 1, m->f32, nf, static_cast<ET*>(L.a2), L.a2_bias, L.head_norm, s.state[r], s.pos, 0, T, m->att, m->max_att, 1, st));
        }
        FX_TRY(plain_linear(L.w_o, W, L.k_o, m->att, m->max_att, m->y));
        pending(L.g1b);
        if (L.d.ff_kind == FLEXLLM_FF_DENSE) {
            a = base(L.w_gu, 2 * L.d.ff, W);
            a.n_split = 2 * L.d.ff; a.glu = 1 + L.d.glu; a.limit = L.d.limit; a.out = m->hid; a.ldo = L.d.ff;
            FX_TRY(norm_linear(a, L.g2));
            FX_TRY(plain_linear(L.w_d, W, L.d.ff, m->hid, L.d.ff, m->y));
            pending(L.g2b);
        } else if (L.d.ff_kind == FLEXLLM_FF_MOE) {
            const int sf = L.d.shared_ff, ldr = L.n_side - 2 * sf;
            a = base(L.w_side, L.n_side, W);
            a.n_split = 2 * sf; a.glu = 1 + L.d.glu; a.limit = L.d.shared_limit; a.out = m->hs; a.ldo = sf; a.out32 = m->route; a.ldo32 = ldr;
            a.h_out = m->hn; a.ldh = W;
            FX_TRY(norm_linear(a, L.g2));
            a = base(L.w_gu, 2 * L.d.ff, W);
            a.w_stride = (size_t)2 * L.d.ff * kw;
            a.n_split = 2 * L.d.ff; a.glu = 1 + L.d.glu; a.limit = L.d.limit; a.out = m->hid; a.ldo = L.d.ff; a.x = m->hn; a.ldx = W;
            a.route = m->route; a.ld_route = ldr; a.experts = L.d.experts; a.top = L.d.top; a.pick = m->pick; a.pick_w = m->pick_w;
            FX_TRY(gemv_float<ET>(a, 2, T, st));
            MoeDownArgs b;
            b.w = L.w_d; b.kpad = pad_k(L.d.ff); b.k = L.d.ff; b.w_stride = (size_t)W * b.kpad; b.h = m->hid; b.ldh = L.d.ff;
            if (sf) { b.ws = L.w_sd; b.ks = sf; b.ks_pad = pad_k(sf); b.hs = m->hs; b.ldhs = sf; }
            b.route = m->route; b.ld_route = ldr; b.experts = L.d.experts; b.top = L.d.top; b.pick = m->pick; b.pick_w = m->pick_w;
            b.y = m->y; b.ldy = W; b.n = W;
            FX_TRY(moe_down_small<ET>(b, T, st));
            pending(L.g2b);
        }
    }
    if (n_want == 1 && T == 1 && !layers_out) {
        GemvArgs a = base(m->head, c.vocab, W);
        a.n_split = 0; a.out32 = logits; a.ldo32 = c.vocab;
        return norm_linear(a, m->g_final);
    }
    if (!n_want && !layers_out) return FLEXLLM_OK;
    FX_TRY(settle());
    if (layers_out) FX_HIP(hipMemcpyAsync(layers_out + (size_t)(runs - 1) * T * W, x, sizeof(float) * T * W, hipMemcpyDeviceToDevice, st));
    if (!n_want) return FLEXLLM_OK;
    FX_HIP(hipMemcpyAsync(m->want, want, sizeof(int) * n_want, hipMemcpyHostToDevice, st));
    RowArgs f;
    f.x = x; f.eps = c.eps; f.width = W; f.rows = n_want; f.rows_src = m->want; f.h = m->hw; f.ldh = W; f.h_f32 = 1; f.g = m->g_final;
    FX_TRY(norm_rows<ET>(f, st));
    GemvArgs a = base(m->head, c.vocab, W);
    a.x = m->hw; a.ldx = W; a.n_split = 0; a.out32 = logits; a.ldo32 = c.vocab;
    return gemv_float<ET>(a, 0, n_want, st);
}

// ---- many tokens --------------------------------------------------------------------------------------------------------
template <typename ET>
static int run_many(flexllm_hybrid* m, HybridSlot& s, const int* tokens, int T, const int* want, int n_want, float* logits, float* layers_out,
                    size_t layer_stride, hipStream_t st) {
    const flexllm_hybrid_config& c = m->cfg;
    const int W = c.width, kw = pad_k(W), ldp = (m->max_et + 7) / 8 * 8, pos0 = s.length;
    FX_TRY(many_workspace<ET>(m, T));
    float* x = m->lx0 ? m->lx0 : m->lx;                   // with a loop, the embedding output stays in lx0
    FX_TRY(embed_rows_bf16(as_bf16(m->embed), c.embed_scale, tokens, T, x, W, c.vocab, &s.pos[3], st));
    RowArgs pend;                                         // what the next row kernel has to take in first
    auto rows_h = [&](const float* g) {
        RowArgs r = pend;
        r.x = x; r.eps = c.eps; r.width = W; r.rows = T;
        if (r.y || r.ys || r.x0) r.x_new = x = m->lx;
        if (g) { r.h = m->lh; r.ldh = kw; r.g = g; }
        pend = RowArgs();
        return norm_rows<ET>(r, st);
    };
    auto gemm = [&](const void* a, int lda, const void* w, int rows, int n, int k) {
        GemmArgs g;
        g.a = a; g.lda = lda; g.w = w; g.m = rows; g.n = n; g.k = pad_k(k);
        return g;
    };
    auto to_y = [&](const void* a, int lda, const void* w, int k) {
        GemmArgs g = gemm(a, lda, w, T, W, k);
        g.n_split = 0; g.y32 = m->ly; g.ldy32 = W;
        return gemm_float<ET>(g, st);
    };
    const int runs = (int)m->runs.size();
    for (int r = 0; r < runs; r++) {
        const HybridLayer& L = m->layers[m->runs[r].layer];
        const int nf = L.n_in - L.n_et, lda = pad_k(L.k_o);
        if (layers_out && r > 0) {
            FX_TRY(rows_h(nullptr));
            FX_HIP(hipMemcpyAsync(layers_out + (size_t)(r - 1) * layer_stride, x, sizeof(float) * T * W, hipMemcpyDeviceToDevice, st));
        }
        if (m->runs[r].again) pend.x0 = m->lx0;
        FX_TRY(rows_h(L.g1));
        GemmArgs g = gemm(m->lh, kw, L.w_in, T, L.n_in, W);
        g.n_split = L.n_et; g.y = m->lproj; g.ldy = ldp; g.y32 = m->lf32; g.ldy32 = nf; g.bias = L.in_bias;
        FX_TRY(gemm_float<ET>(g, st));
        ET *proj = static_cast<ET*>(m->lproj), *att = static_cast<ET*>(m->latt);
        if (L.d.mixer == FLEXLLM_MIX_SHARED_KV) {
            const SharedKvRows<ET> rows = {static_cast<ET*>(s.rows[r]), s.inv_rms[r]};
            FX_TRY(shared_kv_store<ET>(L.sd, m->lf32, nf, rows, s.pos, T, st));
            bool flash = false;
            if constexpr (std::is_same<ET, bf16_t>::value) {
                flash = shared_kv_flash_ok(L.sd);
                if (flash) FX_TRY(shared_kv_flash(L.sd, proj, ldp, L.kv_norm, rows, pos0, T, att, lda, st));
            }
            if (!flash)
                for (int t0 = 0; t0 < T; t0 += kAbsorbTokens) {
                    const int n = T - t0 < kAbsorbTokens ? T - t0 : kAbsorbTokens;
                    FX_TRY(shared_kv_splits<ET>(L.sd, proj + (size_t)t0 * ldp, ldp, nullptr, 0, L.kv_norm, rows, s.pos, t0, n, m->scratch, att + (size_t)t0 * lda, lda, 0, st));
                }
        } else if (L.d.mixer == FLEXLLM_MIX_LATENT) {
            ET *cache = static_cast<ET*>(s.rows[r]), *uk = static_cast<ET*>(L.uk), *uv = static_cast<ET*>(L.uv);
            FX_TRY(latent_store<ET>(L.ld, proj, ldp, nf ? m->lf32 : nullptr, nf, L.latent_norm, L.cos_t, L.sin_t, cache, s.pos, T, st));
            bool flash = false;
            if constexpr (std::is_same<ET, bf16_t>::value) {
                flash = latent_flash_ok(L.ld);
                if (flash) {
                    const int lo = L.d.window > 0 && pos0 - L.d.window + 1 > 0 ? pos0 - L.d.window + 1 : 0;
                    const int rows = pos0 + T - lo, HD = L.d.heads * L.d.dim, HV = L.d.heads * L.d.vdim, ldv = (rows + 63) / 64 * 64;
                    const ET* first = cache + (size_t)lo * L.ld.ldc;
                    GemmArgs k = gemm(first, L.ld.ldc, uk, rows, HD, L.d.kv_rank);
                    k.n_split = HD; k.y = m->lk; k.ldy = HD;
                    FX_TRY(gemm_float<ET>(k, st));
                    GemmArgs v;                                   // transposed: heads x vdim rows of positions
                    v.a = uv; v.lda = L.ld.kvp; v.w = first; v.ldw = L.ld.ldc; v.m = HV; v.n = rows; v.k = L.ld.kvp;
                    v.n_split = rows; v.y = m->lvt; v.ldy = ldv;
                    FX_TRY(gemm_float<ET>(v, st));
                    FX_TRY(latent_flash(L.ld, proj, ldp, static_cast<bf16_t*>(m->lk), HD, static_cast<bf16_t*>(m->lvt), ldv, cache, lo, pos0, T, att, lda, st));
                }
            }
            if (!flash)
                for (int t0 = 0; t0 < T; t0 += kAbsorbTokens) {
                    const int n = T - t0 < kAbsorbTokens ? T - t0 : kAbsorbTokens;
                    FX_TRY(latent_absorbed<ET>(L.ld, proj + (size_t)t0 * ldp, ldp, uk, uv, cache, s.pos, t0, n, m->scratch, att + (size_t)t0 * lda, lda, st));
                }
        } else if (gla_chunks_ok(L.gd)) {
            FX_TRY(gla_chunks<ET>(L.gd, proj, ldp, m->lf32, nf, static_cast<ET*>(L.a2), L.a2_bias, L.head_norm, s.state[r], s.pos, T, m->lgla, att, lda, st));
        } else {
            FX_TRY(gla_steps<ET>(L.gd, proj, ldp, 0, m->lf32, nf, static_cast<ET*>(L.a2), L.a2_bias, L.head_norm, s.state[r], s.pos, 0, T, att, lda, 0, st));
        }
        FX_TRY(to_y(att, lda, L.w_o, L.k_o));
        pend.y = m->ly; pend.ldy = W; pend.gb = L.g1b;
        if (L.d.ff_kind == FLEXLLM_FF_NONE) continue;
        const int kf = pad_k(L.d.ff);
        FX_TRY(rows_h(L.g2));
        if (L.d.ff_kind == FLEXLLM_FF_DENSE) {
            g = gemm(m->lh, kw, L.w_gu, T, 2 * L.d.ff, W);
            g.n_split = 2 * L.d.ff; g.glu = 1 + L.d.glu; g.limit = L.d.limit; g.y = m->lhid; g.ldy = kf;
            FX_TRY(gemm_float<ET>(g, st));
            FX_TRY(to_y(m->lhid, kf, L.w_d, L.d.ff));
            pend.y = m->ly; pend.ldy = W; pend.gb = L.g2b;
            continue;
        }
        const int sf = L.d.shared_ff, ldr = L.n_side - 2 * sf, top = L.d.top, ks = pad_k(sf > 0 ? sf : 1);
        g = gemm(m->lh, kw, L.w_side, T, L.n_side, W);
        g.n_split = 2 * sf; g.glu = 1 + L.d.glu; g.limit = L.d.shared_limit; g.y = m->lhs; g.ldy = ks; g.y32 = m->lroute; g.ldy32 = ldr;
        FX_TRY(gemm_float<ET>(g, st));
        const int tile = gemm_group_tile_rows(T * top / L.d.experts);
        MoePlan p;
        p.pick = m->lpick; p.pick_w = m->lpick_w; p.pos_of = m->lpos_of; p.row_src = m->lrow_src; p.counts = m->lcounts; p.tiles = m->ltiles; p.n_tiles = m->lntiles;
        FX_TRY(moe_plan(m->lroute, ldr, T, L.d.experts, top, tile, p, st));
        // whole tiles plus at most one partial tile per expert, and no more tiles than rows
        int max_tiles = T * top / tile + L.d.experts;
        if (max_tiles > T * top) max_tiles = T * top;
        g = gemm(m->lh, kw, L.w_gu, T * top, 2 * L.d.ff, W);
        g.n_split = 2 * L.d.ff; g.glu = 1 + L.d.glu; g.limit = L.d.limit; g.y = m->lhid; g.ldy = kf;
        g.row_src = m->lrow_src; g.tiles = m->ltiles; g.n_tiles = m->lntiles; g.max_tiles = max_tiles; g.w_stride = (size_t)2 * L.d.ff * kw;
        FX_TRY(gemm_grouped<ET>(g, tile, st));
        g = gemm(m->lhid, kf, L.w_d, T * top, W, L.d.ff);
        g.n_split = 0; g.y32 = m->lys; g.ldy32 = W;
        g.tiles = m->ltiles; g.n_tiles = m->lntiles; g.max_tiles = max_tiles; g.w_stride = (size_t)W * kf;
        FX_TRY(gemm_grouped<ET>(g, tile, st));
        if (sf) {
            FX_TRY(to_y(m->lhs, ks, L.w_sd, sf));
            pend.y = m->ly; pend.route = m->lroute; pend.ld_route = ldr; pend.experts = L.d.experts;
        }
        pend.ldy = W; pend.gb = L.g2b; pend.ys = m->lys; pend.pos_of = m->lpos_of; pend.pick_w = m->lpick_w; pend.top = top;
    }
    if (!n_want && !layers_out) return FLEXLLM_OK;
    FX_TRY(rows_h(nullptr));
    if (layers_out) FX_HIP(hipMemcpyAsync(layers_out + (size_t)(runs - 1) * layer_stride, x, sizeof(float) * T * W, hipMemcpyDeviceToDevice, st));
    if (!n_want) return FLEXLLM_OK;
    FX_HIP(hipMemcpyAsync(m->want, want, sizeof(int) * n_want, hipMemcpyHostToDevice, st));
    for (int r0 = 0; r0 < n_want; r0 += kHeadRows) {
        const int n = n_want - r0 < kHeadRows ? n_want - r0 : kHeadRows;
        RowArgs f;
        f.x = x; f.eps = c.eps; f.width = W; f.rows = n; f.rows_src = m->want + r0; f.g = m->g_final;
        if (n_want <= kSmallTokens) {
            f.h = m->hw; f.ldh = W; f.h_f32 = 1;
            FX_TRY(norm_rows<ET>(f, st));
            GemvArgs a;
            a.w = m->head; a.n = c.vocab; a.k = W; a.kpad = kw; a.x = m->hw; a.ldx = W; a.out32 = logits; a.ldo32 = c.vocab;
            FX_TRY(gemv_float<ET>(a, 0, n, st));
        } else {
            f.h = m->lhead; f.ldh = kw;
            FX_TRY(norm_rows<ET>(f, st));
            GemmArgs g = gemm(m->lhead, kw, m->head, n, c.vocab, W);
            g.n_split = 0; g.y32 = logits + (size_t)r0 * c.vocab; g.ldy32 = c.vocab;
            FX_TRY(gemm_float<ET>(g, st));
        }
    }
    return FLEXLLM_OK;
}

template <typename ET>
static int run_step(flexllm_hybrid* m, int slot, const int* tokens, int n, const int* want, int n_want, float* logits, float* layers_out, hipStream_t st) {
    HybridSlot& s = m->slots[slot];
    const int W = m->cfg.width;
    std::vector<int> part;
    int w0 = 0;
    for (int t0 = 0; t0 < n;) {
        const int T = n - t0 < kPieceTokens ? n - t0 : kPieceTokens;
        part.clear();
        int w1 = w0;
        while (w1 < n_want && want[w1] < t0 + T) part.push_back(want[w1++] - t0);
        float* lg = n_want ? logits + (size_t)w0 * m->cfg.vocab : nullptr;
        if (T <= kSmallTokens && (!layers_out || t0 == 0))
            FX_TRY(run_small<ET>(m, s, tokens + t0, T, part.data(), (int)part.size(), lg, layers_out, st));
        else
            FX_TRY(run_many<ET>(m, s, tokens + t0, T, part.data(), (int)part.size(), lg, layers_out ? layers_out + (size_t)t0 * W : nullptr, (size_t)n * W, st));
        FX_TRY(advance_launch(s.pos, T, st));
        s.length += T;
        w0 = w1;
        t0 += T;
    }
    return FLEXLLM_OK;
}

// One token of the decode loop: *token_io -> logits -> next token, position and step advance on the device.
template <typename ET>
static int decode_token(flexllm_hybrid* m, int slot, int* token_io, const float* rands, int top_k, int* tokens_out, hipStream_t st) {
    HybridSlot& s = m->slots[slot];
    const int zero = 0, V = m->cfg.vocab;
    FX_TRY(run_small<ET>(m, s, token_io, 1, &zero, 1, m->logits, nullptr, st));
    if (top_k == 0) {
        argmax_partial_kernel<<<kArgmaxParts, 256, 0, st>>>(m->logits, V, m->am_v, m->am_i);
        argmax_final_advance_kernel<<<1, 64, 0, st>>>(m->am_v, m->am_i, kArgmaxParts, token_io, tokens_out, s.pos);
    } else {
        TopKOut out = {nullptr, nullptr, nullptr, nullptr, token_io, tokens_out, s.pos};
        topk_partial_kernel<<<kTopKParts, kTopKPartThreads, 0, st>>>(m->logits, V, top_k, m->topk_val, m->topk_idx);
        topk_sample_kernel<256><<<1, 256, 0, st>>>(m->topk_val, m->topk_idx, kTopKParts * top_k, top_k, rands, 1, 1, out);
    }
    FX_LAUNCH_CHECK();
    return FLEXLLM_OK;
}

static int decode_any(flexllm_hybrid* m, int slot, int* token_io, const float* rands, int top_k, int* tokens_out, hipStream_t st) {
    return m->cfg.dtype == 0 ? decode_token<bf16_t>(m, slot, token_io, rands, top_k, tokens_out, st)
                             : decode_token<float>(m, slot, token_io, rands, top_k, tokens_out, st);
}

}  // namespace fx

using namespace fx;

extern "C" {

int flexllm_hybrid_create(flexllm_hybrid** out, const flexllm_hybrid_config* cfg, const flexllm_hybrid_layer* layers,
                          const flexllm_hybrid_weights* w, const flexllm_hybrid_layer_weights* lw) {
    FX_REQUIRE(out && cfg && layers && w && lw, "hybrid_create: null pointer");
    FX_REQUIRE(cfg->layers > 0 && cfg->width > 0 && cfg->width <= 15360 && cfg->vocab > 0 && cfg->max_pos > 0 && cfg->slots > 0 && (cfg->dtype == 0 || cfg->dtype == 1),
               "hybrid_create: layers=%d width=%d vocab=%d max_pos=%d slots=%d dtype=%d", cfg->layers, cfg->width, cfg->vocab, cfg->max_pos, cfg->slots, cfg->dtype);
    FX_REQUIRE(cfg->loop_times == 1 || (cfg->loop_times > 1 && cfg->loop_start >= 0 && cfg->loop_start <= cfg->loop_stop && cfg->loop_stop <= cfg->layers),
               "hybrid_create: layers %d .. %d run %d times", cfg->loop_start, cfg->loop_stop, cfg->loop_times);
    for (int i = 0; i < cfg->layers; i++) FX_TRY(check_layer(*cfg, layers, i));
    flexllm_hybrid* m = new flexllm_hybrid();
    m->cfg = *cfg;
    m->layers.resize(cfg->layers);
    const int start = cfg->loop_times > 1 ? cfg->loop_start : 0, stop = cfg->loop_times > 1 ? cfg->loop_stop : 0;
    for (int i = 0; i < cfg->layers; i++) m->layers[i].d = layers[i];
    for (int i = 0; i < start; i++) m->runs.push_back({i, false});
    for (int k = 0; k < cfg->loop_times; k++)
        for (int i = start; i < stop; i++) m->runs.push_back({i, k > 0 && i == start});
    for (int i = stop; i < cfg->layers; i++) m->runs.push_back({i, false});
    const int rc = cfg->dtype == 0 ? create_model<bf16_t>(m, *w, lw) : create_model<float>(m, *w, lw);
    if (rc) { flexllm_hybrid_destroy(m); return rc; }
    *out = m;
    return FLEXLLM_OK;
}

int flexllm_hybrid_destroy(flexllm_hybrid* m) {
    if (!m) return FLEXLLM_OK;
    (void)hipDeviceSynchronize();
    if (m->graph) (void)hipGraphExecDestroy(m->graph);
    for (void* p : m->pool) (void)hipFree(p);
    for (void* p : m->owned) (void)hipFree(p);
    delete m;
    return FLEXLLM_OK;
}

int flexllm_hybrid_reset(flexllm_hybrid* m, int slot, void* stream) {
    FX_REQUIRE(m && slot >= 0 && slot < m->cfg.slots, "hybrid_reset: slot %d", slot);
    m->slots[slot].length = 0;
    return set_state_launch(m->slots[slot].pos, 0, 0, as_stream(stream));
}

int flexllm_hybrid_length(const flexllm_hybrid* m, int slot, int* length) {
    FX_REQUIRE(m && length && slot >= 0 && slot < m->cfg.slots, "hybrid_length: slot %d", slot);
    *length = m->slots[slot].length;
    return FLEXLLM_OK;
}

int flexllm_hybrid_step(flexllm_hybrid* m, int slot, const int* tokens, int n, const int* want, int n_want, float* logits,
                        float* layers_out, void* stream) {
    FX_REQUIRE(m && tokens && slot >= 0 && slot < m->cfg.slots && n > 0 && n_want >= 0 && (n_want == 0 || (want && logits)), "hybrid_step: slot %d, %d tokens", slot, n);
    FX_REQUIRE(m->slots[slot].length + n <= m->cfg.max_pos, "hybrid_step: %d tokens on top of %d exceed max_pos=%d", n, m->slots[slot].length, m->cfg.max_pos);
    for (int i = 0; i < n_want; i++)
        FX_REQUIRE(want[i] >= 0 && want[i] < n && (i == 0 || want[i] > want[i - 1]), "hybrid_step: want[%d]=%d is not ascending in 0..%d", i, want[i], n - 1);
    hipStream_t st = as_stream(stream);
    return m->cfg.dtype == 0 ? run_step<bf16_t>(m, slot, tokens, n, want, n_want, logits, layers_out, st)
                             : run_step<float>(m, slot, tokens, n, want, n_want, logits, layers_out, st);
}

int flexllm_hybrid_decode(flexllm_hybrid* m, int slot, int* token_io, int steps, const float* rands, int top_k, int* tokens_out,
                          int use_graph, void* stream) {
    FX_REQUIRE(m && token_io && tokens_out && slot >= 0 && slot < m->cfg.slots && steps >= 0, "hybrid_decode: slot %d, %d steps", slot, steps);
    FX_REQUIRE(top_k >= 0 && top_k <= kTopKMax && top_k <= m->cfg.vocab && (top_k == 0 || rands), "hybrid_decode: top_k=%d (0..%d)", top_k, kTopKMax);
    HybridSlot& s = m->slots[slot];
    FX_REQUIRE(s.length + steps <= m->cfg.max_pos, "hybrid_decode: %d steps on top of %d tokens exceed max_pos=%d", steps, s.length, m->cfg.max_pos);
    hipStream_t st = as_stream(stream);
    FX_REQUIRE(!use_graph || st, "hybrid_decode: graph replay needs a non-default stream");
    if (steps == 0) return FLEXLLM_OK;
    FX_TRY(set_state_launch(s.pos, s.length, 0, st));
    if (!use_graph) {
        for (int i = 0; i < steps; i++) FX_TRY(decode_any(m, slot, token_io, rands, top_k, tokens_out, st));
    } else {
        if (!m->graph || m->graph_slot != slot || m->graph_topk != top_k || m->graph_io != token_io || m->graph_out != tokens_out ||
            m->graph_rands != rands || m->graph_stream != st) {
            if (m->graph) { (void)hipGraphExecDestroy(m->graph); m->graph = nullptr; }
            FX_HIP(hipStreamSynchronize(st));
            hipGraph_t graph;
            FX_HIP(hipStreamBeginCapture(st, hipStreamCaptureModeThreadLocal));
            const int rc = decode_any(m, slot, token_io, rands, top_k, tokens_out, st);
            hipError_t e = hipStreamEndCapture(st, &graph);
            if (rc) { if (e == hipSuccess) (void)hipGraphDestroy(graph); return rc; }
            FX_HIP(e);
            e = hipGraphInstantiate(&m->graph, graph, nullptr, nullptr, 0);
            (void)hipGraphDestroy(graph);
            if (e != hipSuccess) m->graph = nullptr;
            FX_HIP(e);
            m->graph_slot = slot; m->graph_topk = top_k; m->graph_io = token_io; m->graph_out = tokens_out; m->graph_rands = rands; m->graph_stream = st;
        }
        for (int i = 0; i < steps; i++) FX_HIP(hipGraphLaunch(m->graph, st));
    }
    s.length += steps;
    return FLEXLLM_OK;
}

int flexllm_hybrid_generate(flexllm_hybrid* m, int slot, const int* prompt, int n_prompt, int steps, const float* rands, int top_k,
                            int* tokens_out, int use_graph, void* stream) {
    FX_REQUIRE(m && prompt && tokens_out && n_prompt >= 1 && slot >= 0 && slot < m->cfg.slots, "hybrid_generate: slot %d, prompt of %d", slot, n_prompt);
    if (n_prompt > 1) FX_TRY(flexllm_hybrid_step(m, slot, prompt, n_prompt - 1, nullptr, 0, nullptr, nullptr, stream));
    copy_int_kernel<<<1, 1, 0, as_stream(stream)>>>(prompt + n_prompt - 1, m->gen_token);
    FX_LAUNCH_CHECK();
    return flexllm_hybrid_decode(m, slot, m->gen_token, steps, rands, top_k, tokens_out, use_graph, stream);
}

int flexllm_hybrid_check(flexllm_hybrid* m) {
    FX_REQUIRE(m, "hybrid_check: null pointer");
    FX_HIP(hipDeviceSynchronize());
    for (size_t i = 0; i < m->slots.size(); i++) {
        int st[4] = {0, 0, 0, 0};
        FX_HIP(hipMemcpy(st, m->slots[i].pos, sizeof(st), hipMemcpyDeviceToHost));
        if (st[3]) {
            (void)hipMemset(&m->slots[i].pos[3], 0, sizeof(int));
            set_error("slot %zu: a token id outside the vocabulary (%d entries) was fed in; token 0 was used instead", i, m->cfg.vocab);
            return FLEXLLM_EINVAL;
        }
    }
    return FLEXLLM_OK;
}

}  // extern "C"
