// Models of described layers: a list of layer descriptions (mixer, sizes, feed-forward) run in order, a range of them
// possibly several times, each pass with its own cache or state.  The model is an axq_model: its tokens, positions,
// history, sampling, graphs and generation are those of axq_decode.hip, which calls the step and the rows here.
//
// A decode step is three kernels per recurrent layer (projections with the norm in front and the activations behind;
// state update; output projection with the gated norm in front and the residual add behind) and four plus two for
// attention with a feed-forward.  In a parallel layer the first products of mixer and feed-forward are one launch and their
// last ones are one product over the inputs in a row.  A prompt's rows take the same mechanisms in their row form: a norm or
// gate pass that writes the product's operand, one product launch for all projections that read it, the recurrence or attention.
// The residual stream, norms, scores, routers, states and everything that enters a recurrence beyond the projections are f32.
#include <math.h>

#include <map>
#include <new>
#include <string>
#include <vector>

#include "axq_dense.h"
#include "axq_model.h"

namespace {

struct Slot {
    bool linear = false;
    int64_t rows = 0, cols = 0;
    axq_weight *w = nullptr;   // linear
    float *v = nullptr;        // vector, on the device
    std::vector<float> host;   // vector, a copy
    bool set = false;
    axq_weight *into = nullptr; // linear: kept as rows row0 .. of this one, or
    int64_t row0 = 0;
    bool spread = false;        // ... group by group of AXQ_GLU_GROUP rows, every second group
};

struct Layer {
    axq_layer_config c;
    std::map<std::string, Slot> t;
    float *bias = nullptr; // attention: [heads][nt]
    int nt = 1;
    bool bias_ready = false;
    float *temp = nullptr; // attention: [cache positions]
    std::map<std::string, axq_weight *> fused; // what linears with Slot::into are kept in
    const float *rc = nullptr, *rs = nullptr;  // softmax attention: rotation by position
};

// Cosines and sines by position, shared by the layers that rotate alike
struct Rotation {
    axq_layer_config c;
    float *rc = nullptr, *rs = nullptr;
};

struct Run {
    int layer;
    void *kc = nullptr, *vc = nullptr, *pkc = nullptr, *pvc = nullptr;
    float *state = nullptr, *prev = nullptr;
};

} // namespace

struct axq_stack {
    axq_stack_config c;
    bool f32;
    std::vector<Layer> layers;
    Layer top; // pos, final.norm, head
    std::vector<Run> runs;
    std::vector<Rotation> rotations;
    // activations of a step
    float *proj = nullptr, *o = nullptr, *z = nullptr, *part = nullptr;
    float *past = nullptr; // mean over the layers: the embedding and every layer's result
    float *ez = nullptr, *wt = nullptr; // mixture: the chosen experts' inner activations and weights
    int32_t *sel = nullptr;
    void *qs = nullptr;
    // activations of `cap` rows
    int cap = 0;
    float *r_h = nullptr, *r_proj = nullptr, *r_o = nullptr, *r_z = nullptr, *r_logits = nullptr;
    float *r_seg = nullptr, *r_segw = nullptr; // segments of a recurrence
    void *r_x = nullptr, *r_qs = nullptr;
    void *r_x2 = nullptr, *r_f = nullptr; // operands: the second norm of a parallel layer; what goes into a feed-forward's last product
    float *r_past = nullptr;              // mean over the layers
    void *r_ez = nullptr;                 // mixture: by slot, the operands of the experts' last products,
    float *r_ey = nullptr, *r_wt = nullptr; // ... their results; by row, the weights
    int32_t *r_route = nullptr;           // ... and the chosen experts, slots, rows by slot and tiles
    int32_t *r_want = nullptr;
    int logits_cap = 0;
    float *trace = nullptr;
    int trace_total = 0, trace_row0 = 0;
};

namespace {

constexpr int LOGITS_ROWS = 256; // wanted rows per pass through the head
inline int pad64(int k) { return (k + 63) / 64 * 64; }

void add_slot(Layer &l, const char *name, bool linear, int64_t rows, int64_t cols) {
    Slot s;
    s.linear = linear;
    s.rows = rows;
    s.cols = cols;
    l.t[name] = s;
}

void add_norm(Layer &l, const std::string &name, int64_t width, int kind) {
    add_slot(l, name.c_str(), false, 1, width);
    if (kind == AXQ_NORM_LAYER) return;
    add_slot(l, (name + ".b").c_str(), false, 1, width);
    add_slot(l, (name + ".alpha").c_str(), false, 1, 1);
}

int mixer_out(const axq_layer_config &c) { return c.heads * (c.mixer == AXQ_MIX_WKV ? c.dim : c.vdim); }

// A layer's first products, in launch order: those of its mixer, those of its feed-forward.
struct First {
    const char *name;
    int act;
    int width;
    const char *mu;
};

std::vector<First> mixer_firsts(const axq_layer_config &c) {
    const int q = c.heads * c.dim, v = c.heads * c.vdim;
    switch (c.mixer) {
    case AXQ_MIX_ATTENTION:
        return {{"mix.q", AXQ_ACT_NONE, q, nullptr}, {"mix.k", AXQ_ACT_NONE, c.kv_heads * c.dim, nullptr}, {"mix.v", AXQ_ACT_NONE, c.kv_heads * c.vdim, nullptr}};
    case AXQ_MIX_SOFTMAX: {
        std::vector<First> f = {{"mix.q", AXQ_ACT_NONE, q, nullptr}, {"mix.k", AXQ_ACT_NONE, c.kv_heads * c.dim, nullptr}};
        if (!c.keys_as_values) f.push_back({"mix.v", AXQ_ACT_NONE, c.kv_heads * c.vdim, nullptr});
        if (c.head_gate) f.push_back({"mix.g", AXQ_ACT_SIGMOID, c.heads, nullptr});
        return f;
    }
    case AXQ_MIX_LIGHTNING:
        return {{"mix.q", AXQ_ACT_SILU, q, nullptr}, {"mix.k", AXQ_ACT_SILU, q, nullptr}, {"mix.v", AXQ_ACT_SILU, v, nullptr}, {"mix.g", AXQ_ACT_SIGMOID, v, nullptr}};
    default:
        return {{"mix.r", AXQ_ACT_NONE, q, "mix.mu.r"}, {"mix.k", AXQ_ACT_NONE, q, "mix.mu.k"}, {"mix.v", AXQ_ACT_NONE, q, "mix.mu.v"},
                {"mix.g", AXQ_ACT_SILU, q, "mix.mu.g"}, {"mix.w1", AXQ_ACT_TANH, pad64(c.decay_rank), "mix.mu.w"}};
    }
}

int glu_rows(int ff) { return (ff + AXQ_GLU_GROUP - 1) / AXQ_GLU_GROUP * 2 * AXQ_GLU_GROUP; }

std::vector<First> ff_firsts(const axq_layer_config &c) {
    if (c.ff <= 0) return {};
    switch (c.ff_kind) {
    case AXQ_FF_GLU: return {{"mlp.gu", AXQ_ACT_GLU_GELU, glu_rows(c.ff), nullptr}};
    case AXQ_FF_MOE: {
        std::vector<First> f = {{"mlp.router", AXQ_ACT_NONE, c.experts, nullptr}};
        if (c.shared_ff > 0) {
            f.push_back({"mlp.shared.sg", AXQ_ACT_SIGMOID, 1, nullptr});
            f.push_back({"mlp.shared.up", AXQ_ACT_RELU2, pad64(c.shared_ff), nullptr});
        }
        return f;
    }
    default: return {{"mlp.up", AXQ_ACT_NONE, c.ff, nullptr}};
    }
}

size_t total_width(const std::vector<First> &f) {
    size_t n = 0;
    for (const First &x : f) n += x.width;
    return n;
}

// floats per row of a mixer's first products (time mixing: and of its decays)
size_t proj_width(const axq_layer_config &c) { return total_width(mixer_firsts(c)) + (c.mixer == AXQ_MIX_WKV ? (size_t)c.heads * c.dim : 0); }

template <class T>
hipError_t dev_alloc(T **p, size_t bytes) { return hipMalloc((void **)p, bytes ? bytes : 16); }

// Bucket of a key n tokens back: exact below rows / 2, then logarithmic up to `dmax`.  A quotient that is an integer in
// exact arithmetic must not fall below it by rounding.
int distance_bucket(int n, int rows, int dmax) {
    const int half = rows / 2;
    if (n < half) return n;
    if (dmax <= half) return rows - 1;
    const double v = log((double)n / half) / log((double)dmax / half) * (rows - half), near = nearbyint(v);
    const int b = half + (int)(fabs(v - near) < 1e-9 ? near : floor(v));
    return b < rows - 1 ? b : rows - 1;
}

int build_bias(axq_model *m, Layer &l) {
    axq_ctx *ctx = m->ctx;
    const axq_layer_config &c = l.c;
    const int cap = m->cfg.max_position_embeddings;
    l.nt = 1;
    if (c.bias_rows > 0) {
        while (l.nt < cap && distance_bucket(l.nt - 1, c.bias_rows, c.bias_max) < c.bias_rows - 1) l.nt++;
    }
    std::vector<float> b((size_t)c.heads * l.nt);
    const std::vector<float> &pb = l.t["mix.pb"].host;
    for (int h = 0; h < c.heads; h++)
        for (int n = 0; n < l.nt; n++)
            b[(size_t)h * l.nt + n] = pb[h] + (c.bias_rows > 0 ? l.t["mix.rel"].host[(size_t)distance_bucket(n, c.bias_rows, c.bias_max) * c.heads + h] : 0.f);
    AXQ_HIP(ctx, hipStreamSynchronize(ctx->stream), AXQ_ERR_DRIVER);
    if (l.bias) (void)hipFree(l.bias);
    l.bias = nullptr;
    axq_model_drop_graphs(m);
    AXQ_HIP(ctx, dev_alloc(&l.bias, b.size() * 4), AXQ_ERR_ALLOCATION_FAILED);
    AXQ_HIP(ctx, hipMemcpy(l.bias, b.data(), b.size() * 4, hipMemcpyHostToDevice), AXQ_ERR_COPY_FAILED);
    l.bias_ready = true;
    return AXQ_OK;
}

// A vector on the device; NULL where the layer has none of that name.
float *vec(Layer &l, const char *name) {
    auto it = l.t.find(name);
    return it == l.t.end() ? nullptr : it->second.v;
}

axq_in norm_in(const axq_stack &s, Layer &l, const std::string &name, const float *x) {
    axq_in in;
    in.x = x;
    in.k = s.c.width;
    in.eps = s.c.norm_eps;
    in.nw = vec(l, name.c_str());
    if (s.c.norm == AXQ_NORM_LAYER) return in;
    in.alpha = vec(l, (name + ".alpha").c_str());
    in.nb = vec(l, (name + ".b").c_str());
    return in;
}

int norm_mode(const axq_stack &s) { return s.c.norm == AXQ_NORM_LAYER ? AXQ_IN_LAYER_NORM : AXQ_IN_TANH_NORM; }

int norm_rows(axq_ctx *ctx, const axq_stack &s, const axq_in &in, int m, axq_rows_out out) {
    if (s.c.norm == AXQ_NORM_LAYER) return axq_rows_layer_norm(ctx, in, m, in.nw, out, nullptr, out);
    return axq_rows_tanh_norm(ctx, in, m, true, 0, nullptr, out);
}

const axq_weight *weight_of(Layer &l, const char *name) {
    auto it = l.fused.find(name);
    return it != l.fused.end() ? it->second : l.t[name].w;
}

axq_part part_of(Layer &l, const char *name, int act, void *y, int ldy, const float *resid = nullptr) {
    const axq_weight *w = weight_of(l, name);
    axq_part p = {};
    p.w = reinterpret_cast<const uint16_t *>(w->codes);
    p.ldw = (int)(w->codes_pitch / 2);
    p.n = (int)w->n_rows;
    p.act = act;
    p.y = y;
    p.ldy = ldy;
    p.resid = resid;
    return p;
}

axq_seg seg_of(Layer &l, const char *name, const float *x, int k) {
    const axq_weight *w = weight_of(l, name);
    axq_seg g = {};
    g.w = reinterpret_cast<const uint16_t *>(w->codes);
    g.ldw = (int)(w->codes_pitch / 2);
    g.k = k;
    g.count = 1;
    g.x = x;
    return g;
}

// First products over `m` rows; product i's results are a block [m][f[i].width] of buf (out[i]).
struct Proj {
    axq_parts parts = {};
    std::vector<First> f;
    std::vector<float *> out;
    int width(int i) const { return f[i].width; }
};

void add_firsts(Proj &p, Layer &l, const std::vector<First> &f, float *buf, int m, const float *nw) {
    for (const First &x : f) {
        axq_part &q = p.parts.p[p.parts.n_parts++];
        q = part_of(l, x.name, x.act, buf, x.width);
        if (x.mu) q.mu = vec(l, x.mu);
        q.nw = nw;
        p.f.push_back(x);
        p.out.push_back(buf);
        buf += (size_t)x.width * m;
    }
    p.out.push_back(buf); // behind the last one
}

axq_sig_attn attn_of(const axq_stack &s, Layer &l, const Run &r, int cap) {
    axq_sig_attn a;
    a.heads = l.c.heads; a.kv_heads = l.c.kv_heads; a.dim = l.c.dim; a.vdim = l.c.vdim;
    a.cap = cap;
    a.scale = l.c.scale; a.eps = s.c.norm_eps;
    a.qn = vec(l, "mix.q.norm"); a.kn = vec(l, "mix.k.norm");
    a.temp = l.temp; a.bias = l.bias; a.nt = l.nt;
    a.kc = r.kc; a.vc = r.vc;
    a.f32 = s.f32;
    return a;
}

axq_soft_attn soft_attn_of(const axq_stack &s, const Layer &l, const Run &r, int cap) {
    axq_soft_attn a = {};
    a.heads = l.c.heads; a.kv_heads = l.c.kv_heads; a.dim = l.c.dim; a.vdim = l.c.vdim;
    a.cap = cap;
    a.window = l.c.window > 0 ? l.c.window : cap;
    a.pool = l.c.window > 0 ? l.c.pool : 0;
    a.scale = l.c.scale;
    a.rot_dims = l.c.rot_dims;
    a.rc = l.rc; a.rs = l.rs;
    a.kc = r.kc; a.vc = r.vc; a.pkc = r.pkc; a.pvc = r.pvc;
    a.f32 = s.f32;
    return a;
}

// The projections that softmax attention reads
struct SoftIn { const float *q, *k, *v, *gate; int ldq, ldk, ldv; };
SoftIn soft_in(const axq_layer_config &c, const Proj &p) {
    const int v = c.keys_as_values ? 1 : 2;
    return {p.out[0], p.out[1], p.out[v], c.head_gate ? p.out[v + 1] : nullptr, p.width(0), p.width(1), p.width(v)};
}

axq_moe_router router_of(const axq_layer_config &c) { return {c.experts, c.top, c.groups, c.groups_keep}; }

axq_linstate linstate_of(Layer &l, const Run &r, const Proj &p, float *o) {
    axq_linstate a = {};
    const axq_layer_config &c = l.c;
    a.heads = c.heads;
    a.dk = c.dim;
    a.dv = c.mixer == AXQ_MIX_WKV ? c.dim : c.vdim;
    a.q = p.out[0]; a.k = p.out[1]; a.v = p.out[2];
    a.ldq = p.width(0); a.ldk = p.width(1); a.ldv = p.width(2);
    if (c.mixer == AXQ_MIX_LIGHTNING) a.decay = vec(l, "mix.decay");
    else a.u = vec(l, "mix.u");
    a.state = r.state;
    a.o = o;
    return a;
}

// The integers of a mixture's rows: chosen experts, slots, rows by slot, tiles.
struct Route { int32_t *sel, *slot_of, *src, *tiles; int bm, max_tiles; };
Route route_of(const axq_stack &s, const axq_layer_config &c, int m) {
    Route r;
    const int n = m * c.top;
    r.sel = s.r_route;
    r.slot_of = r.sel + n;
    r.src = r.slot_of + n;
    r.tiles = r.src + n;
    r.bm = axq_dense_gemm_rows_per_tile(n, c.experts, s.f32);
    r.max_tiles = axq_moe_max_tiles(n, c.experts, r.bm);
    return r;
}

int reserve_rows(axq_model *m, int rows) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    if (rows <= s.cap) return AXQ_OK;
    int cap = 64;
    while (cap < rows) cap *= 2;
    AXQ_HIP(ctx, hipStreamSynchronize(ctx->stream), AXQ_ERR_DRIVER);
    for (void **p : {(void **)&s.r_h, (void **)&s.r_proj, (void **)&s.r_o, (void **)&s.r_z, (void **)&s.r_seg, (void **)&s.r_segw, &s.r_x, &s.r_qs,
                     &s.r_x2, &s.r_f, (void **)&s.r_past, &s.r_ez, (void **)&s.r_ey, (void **)&s.r_wt, (void **)&s.r_route}) {
        if (*p) (void)hipFree(*p);
        *p = nullptr;
    }
    s.cap = 0;
    size_t proj = 0, o = 0, z = 0, x = pad64(s.c.width), f = 0, qs = 0, seg = 0, segw = 0, ez = 0, wt = 0, route = 0;
    auto most = [](size_t &a, size_t b) { a = b > a ? b : a; };
    for (Layer &l : s.layers) {
        most(proj, proj_width(l.c));
        const size_t mo = mixer_out(l.c);
        most(o, mo);
        most(z, total_width(ff_firsts(l.c)));
        most(x, pad64((int)mo));
        if (l.c.mixer == AXQ_MIX_WKV) most(x, (size_t)5 * pad64(s.c.width));
        if (l.c.ff > 0) most(f, pad64(l.c.ff_kind == AXQ_FF_MOE ? l.c.shared_ff : l.c.ff));
        if (l.c.ff > 0 && l.c.ff_kind == AXQ_FF_MOE) {
            most(ez, (size_t)l.c.top * pad64(l.c.ff));
            most(wt, l.c.top);
            most(route, (size_t)cap * l.c.top * 3 + 4 + 4 * ((size_t)cap * l.c.top / 64 + 1 + l.c.experts));
        }
        if (l.c.mixer == AXQ_MIX_ATTENTION) {
            axq_sig_attn a = {};
            a.heads = l.c.heads; a.dim = l.c.dim; a.f32 = s.f32;
            most(qs, axq_sig_attn_q_bytes(a, 1));
        } else if (l.c.mixer == AXQ_MIX_SOFTMAX) {
            axq_soft_attn a = {};
            a.heads = l.c.heads; a.dim = l.c.dim; a.f32 = s.f32;
            most(qs, axq_soft_attn_q_bytes(a, 1));
        } else {
            const size_t w = (size_t)l.c.heads * l.c.dim;
            most(seg, w * (l.c.mixer == AXQ_MIX_WKV ? l.c.dim : l.c.vdim));
            most(segw, w);
        }
    }
    const size_t es = s.f32 ? 4 : 2, W = s.c.width, C = cap;
    hipError_t e = dev_alloc(&s.r_h, C * W * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_proj, C * proj * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_o, C * o * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_z, C * z * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_x, C * x * es);
    if (e == hipSuccess) e = dev_alloc(&s.r_f, C * f * es);
    if (e == hipSuccess) e = dev_alloc(&s.r_qs, C * qs);
    if (e == hipSuccess) e = dev_alloc(&s.r_seg, seg * AXQ_LINSTATE_SEGS * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_segw, segw * AXQ_LINSTATE_SEGS * 4);
    if (e == hipSuccess && s.c.parallel) e = dev_alloc(&s.r_x2, C * pad64(s.c.width) * es);
    if (e == hipSuccess && s.c.depth_average) e = dev_alloc(&s.r_past, (s.runs.size() + 1) * C * W * 4);
    if (e == hipSuccess && wt) {
        e = dev_alloc(&s.r_ez, C * ez * es);
        if (e == hipSuccess) e = dev_alloc(&s.r_ey, C * wt * W * 4);
        if (e == hipSuccess) e = dev_alloc(&s.r_wt, C * wt * 4);
        if (e == hipSuccess) e = dev_alloc(&s.r_route, route * 4);
    }
    if (e != hipSuccess) return axq_fail(ctx, AXQ_ERR_ALLOCATION_FAILED, "activations for %d rows: %s", cap, hipGetErrorString(e));
    s.cap = cap;
    return AXQ_OK;
}

// The result of a layer, `y` (of the residual stream `x`), and the mean over the layers' results that follows it.
axq_avg avg_of(const axq_stack &s, Layer &l, const float *past, size_t stride, size_t run, float *out) {
    axq_avg a = {};
    if (!s.c.depth_average) return a;
    a.w = vec(l, "dwa");
    a.past = past;
    a.stride = stride;
    a.n = (int)run + 1;
    a.out = out;
    return a;
}

// Between a feed-forward's first and last products, one token: a mixture chooses its experts and takes their first ones.
// ff: its first products, of norm2(x); in: that norm.  Then its last products are the segments added to `out`.
int ff_token(axq_ctx *ctx, axq_stack &s, Layer &l, float *const *ff, const axq_in &in, axq_in &out) {
    const axq_layer_config &c = l.c;
    if (c.ff_kind == AXQ_FF_GLU) {
        axq_seg &g = out.seg[out.n_seg++];
        g = seg_of(l, "mlp.down", ff[0], c.ff);
        g.glu = 1;
        return AXQ_OK;
    }
    int rc;
    if ((rc = axq_moe_route(ctx, router_of(c), ff[0], c.experts, 1, s.sel, s.wt))) return rc;
    axq_parts up = {};
    up.n_parts = 1;
    up.p[0] = part_of(l, "mlp.experts.up", AXQ_ACT_RELU2, s.ez, 0);
    up.p[0].n = c.top * c.ff;
    up.p[0].nw = in.nw;
    up.p[0].sel = s.sel;
    up.p[0].sel_rows = c.ff;
    if ((rc = axq_dense_gemv(ctx, AXQ_IN_LAYER_NORM, in, up))) return rc;
    if (c.shared_ff > 0) {
        axq_seg &g = out.seg[out.n_seg++];
        g = seg_of(l, "mlp.shared.down", ff[2], c.shared_ff);
        g.scale = ff[1];
    }
    axq_seg &g = out.seg[out.n_seg++];
    g = seg_of(l, "mlp.experts.down", s.ez, c.ff);
    g.count = c.top;
    g.ldx = c.ff;
    g.stride = (size_t)s.c.width * g.ldw;
    g.sel = s.sel;
    g.scale = s.wt;
    return AXQ_OK;
}

// A feed-forward's last products over rows: y += .., with the first ones' results in ff and h the operand they read.
int ff_rows(axq_ctx *ctx, axq_stack &s, Layer &l, float *const *ff, const void *h, int nb, float *y, const axq_avg &avg) {
    const axq_layer_config &c = l.c;
    const int W = s.c.width, ldw = pad64(W);
    int rc;
    axq_parts d = {};
    d.n_parts = 1;
    if (c.ff_kind != AXQ_FF_MOE) {
        const int ldf = pad64(c.ff);
        const axq_rows_out f = {s.r_f, ldf, s.f32};
        if (c.ff_kind == AXQ_FF_POLY) {
            axq_in zin;
            zin.x = ff[0];
            zin.k = c.ff;
            zin.eps = s.c.norm_eps;
            zin.coef = vec(l, "mlp.act");
            if ((rc = axq_rows_poly_norm(ctx, zin, nb, f))) return rc;
        } else if (s.f32) {
            if ((rc = axq_rows_glu(ctx, ff[0], glu_rows(c.ff), c.ff, nb, f))) return rc;
        } else if ((rc = axq_rows_zero_tail(ctx, nb, c.ff, f))) {
            return rc;
        }
        d.p[0] = part_of(l, "mlp.down", AXQ_ACT_NONE, y, W, y);
        d.p[0].x = s.r_f;
        d.p[0].avg = avg;
        return axq_dense_gemm(ctx, d, nb, c.ff, ldf, s.f32);
    }
    if (c.shared_ff > 0) {
        const int lds = pad64(c.shared_ff);
        if ((rc = axq_rows_zero_tail(ctx, nb, c.shared_ff, {s.r_f, lds, s.f32}))) return rc;
        d.p[0] = part_of(l, "mlp.shared.down", AXQ_ACT_NONE, y, W, y);
        d.p[0].x = s.r_f;
        d.p[0].scale = ff[1];
        if ((rc = axq_dense_gemm(ctx, d, nb, c.shared_ff, lds, s.f32))) return rc;
    }
    const Route r = route_of(s, c, nb);
    const int n = nb * c.top, ldf = pad64(c.ff);
    if ((rc = axq_moe_route(ctx, router_of(c), ff[0], c.experts, nb, r.sel, s.r_wt))) return rc;
    if ((rc = axq_moe_sort(ctx, r.sel, n, c.top, c.experts, r.bm, r.slot_of, r.src, r.tiles))) return rc;
    axq_part p = part_of(l, "mlp.experts.up", AXQ_ACT_RELU2, s.r_ez, ldf);
    axq_groups g = {r.tiles, r.src, (size_t)c.ff * p.ldw, r.max_tiles, r.bm};
    p.n = c.ff;
    p.out16 = !s.f32;
    p.x = h;
    if ((rc = axq_dense_gemm_grouped(ctx, p, g, W, ldw, s.f32))) return rc;
    if ((rc = axq_rows_zero_tail(ctx, n, c.ff, {s.r_ez, ldf, s.f32}))) return rc;
    p = part_of(l, "mlp.experts.down", AXQ_ACT_NONE, s.r_ey, W);
    g.src = nullptr;
    g.stride = (size_t)W * p.ldw;
    p.n = W;
    p.x = s.r_ez;
    if ((rc = axq_dense_gemm_grouped(ctx, p, g, c.ff, ldf, s.f32))) return rc;
    return axq_moe_combine(ctx, s.r_ey, r.slot_of, s.r_wt, c.top, nb, W, y, avg);
}

// Where rows' first products of a feed-forward go that are operands of its last ones
void ff_operands(const axq_stack &s, const axq_layer_config &c, Proj &p, int first) {
    for (int i = first; i < p.parts.n_parts; i++) {
        axq_part &q = p.parts.p[i];
        const bool glu = q.act == AXQ_ACT_GLU_GELU && !s.f32, shared = c.ff_kind == AXQ_FF_MOE && q.act == AXQ_ACT_RELU2;
        if (!glu && !shared) continue;
        q.y = s.r_f;
        q.ldy = pad64(glu ? c.ff : c.shared_ff);
        q.out16 = !s.f32;
    }
}

} // namespace

int axq_stack_layer_runs(const axq_model *m) { return (int)m->stack->runs.size(); }

bool axq_stack_recurrent(const axq_model *m) {
    for (const Layer &l : m->stack->layers)
        if (l.c.mixer != AXQ_MIX_ATTENTION && l.c.mixer != AXQ_MIX_SOFTMAX) return true;
    return false;
}

void axq_stack_trace(axq_model *m, float *layers, int total_rows, int row0) {
    m->stack->trace = layers;
    m->stack->trace_total = total_rows;
    m->stack->trace_row0 = row0;
}

int axq_stack_ready(axq_model *m) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    if (!m->emb && !m->emb32) return axq_fail(ctx, AXQ_ERR_INVALID_DATA, "Invalid quantized data: embedding not set");
    for (auto &kv : s.top.t)
        if (!kv.second.set) return axq_fail(ctx, AXQ_ERR_INVALID_DATA, "Invalid quantized data: %s not set", kv.first.c_str());
    for (size_t i = 0; i < s.layers.size(); i++) {
        Layer &l = s.layers[i];
        for (auto &kv : l.t)
            if (!kv.second.set) return axq_fail(ctx, AXQ_ERR_INVALID_DATA, "Invalid quantized data: %s of layer %d not set", kv.first.c_str(), (int)i);
        int rc;
        if (l.c.mixer == AXQ_MIX_ATTENTION && !l.bias_ready && (rc = build_bias(m, l))) return rc;
    }
    return AXQ_OK;
}

int axq_stack_step(axq_model *m) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    const int W = s.c.width;
    const bool average = s.c.depth_average && !s.runs.empty();
    float *x = average ? s.past : m->h;
    int rc;
    if ((rc = axq_rows_embed(ctx, m->emb, m->emb32, vec(s.top, "pos"), m->tok, m->pos, 0, 1, W, x))) return rc;
    for (size_t run = 0; run < s.runs.size(); run++) {
        Run &r = s.runs[run];
        Layer &l = s.layers[r.layer];
        const axq_layer_config &c = l.c;
        float *y = average ? s.past + (run + 1) * W : m->h; // the layer's result
        const axq_avg avg = avg_of(s, l, s.past, W, run, m->h);
        const bool parallel = s.c.parallel && c.ff > 0;
        axq_in in = norm_in(s, l, "norm1", x), out_in;
        Proj p;
        add_firsts(p, l, mixer_firsts(c), s.proj, 1, in.nw);
        float *const *ff = nullptr;
        if (parallel) {
            p.out.reserve(p.out.size() + 8);
            ff = p.out.data() + p.out.size();
            add_firsts(p, l, ff_firsts(c), s.z, 1, vec(l, "norm2"));
        }
        int out_mode = AXQ_IN_PLAIN;
        in.prev = r.prev;
        in.pos = m->pos;
        if ((rc = axq_dense_gemv(ctx, c.mixer == AXQ_MIX_WKV ? AXQ_IN_TANH_NORM_MIX : norm_mode(s), in, p.parts))) return rc;
        out_in.x = s.o;
        out_in.k = mixer_out(c);
        out_in.eps = s.c.norm_eps;
        if (c.mixer == AXQ_MIX_ATTENTION) {
            const axq_sig_attn a = attn_of(s, l, r, m->cfg.max_position_embeddings);
            if ((rc = axq_sig_attn_token(ctx, a, p.out[0], p.out[1], p.out[2], m->pos, s.qs, s.part, s.o))) return rc;
        } else if (c.mixer == AXQ_MIX_SOFTMAX) {
            const axq_soft_attn a = soft_attn_of(s, l, r, m->cfg.max_position_embeddings);
            const SoftIn i = soft_in(c, p);
            if ((rc = axq_soft_attn_token(ctx, a, i.q, i.k, i.v, i.gate, m->pos, s.qs, s.part, s.o))) return rc;
        } else {
            axq_linstate_step st = {};
            st.a = linstate_of(l, r, p, s.o);
            st.pos = m->pos;
            if (c.mixer == AXQ_MIX_WKV) {
                const axq_weight *w2 = l.t["mix.w2"].w;
                st.t1 = p.out[4];
                st.w2 = reinterpret_cast<const uint16_t *>(w2->codes);
                st.ldw2 = (int)(w2->codes_pitch / 2);
                st.rank = c.decay_rank;
                st.w0 = vec(l, "mix.w0");
                st.norm_w = vec(l, "mix.norm");
                st.gate = p.out[3];
                st.eps = s.c.norm_eps;
                st.prev_in = in;
                st.prev = r.prev;
            } else {
                out_mode = AXQ_IN_RMS_GATE;
                out_in.nw = vec(l, "mix.norm");
                out_in.gate = p.out[3];
            }
            if ((rc = axq_linstate_token(ctx, st))) return rc;
        }
        axq_in last; // the layer's last product: the feed-forward's, in a parallel layer with the mixer's in front
        if (parallel && out_mode == AXQ_IN_PLAIN) {
            last.seg[last.n_seg++] = seg_of(l, "mix.o", s.o, mixer_out(c));
        } else {
            axq_parts o = {};
            o.n_parts = 1;
            o.p[0] = part_of(l, "mix.o", AXQ_ACT_NONE, y, W, x);
            if (c.ff <= 0) o.p[0].avg = avg;
            if ((rc = axq_dense_gemv(ctx, out_mode, out_in, o))) return rc;
        }
        if (c.ff > 0) {
            const float *resid = last.n_seg ? x : y;
            axq_in in2 = norm_in(s, l, "norm2", parallel ? x : y);
            Proj f;
            if (!parallel) {
                add_firsts(f, l, ff_firsts(c), s.z, 1, in2.nw);
                ff = f.out.data();
                if ((rc = axq_dense_gemv(ctx, norm_mode(s), in2, f.parts))) return rc;
            }
            axq_parts d = {};
            d.n_parts = 1;
            d.p[0] = part_of(l, c.ff_kind == AXQ_FF_MOE ? "mix.o" : "mlp.down", AXQ_ACT_NONE, y, W, resid); // segments bring their own weights
            d.p[0].avg = avg;
            int mode = AXQ_IN_SEGMENTS;
            if (c.ff_kind == AXQ_FF_POLY) {
                mode = AXQ_IN_POLY_NORM;
                last.x = ff[0];
                last.k = c.ff;
                last.eps = s.c.norm_eps;
                last.coef = vec(l, "mlp.act");
            } else if ((rc = ff_token(ctx, s, l, ff, in2, last))) {
                return rc;
            }
            if ((rc = axq_dense_gemv(ctx, mode, last, d))) return rc;
        }
        x = m->h;
    }
    axq_parts hd = {};
    hd.n_parts = 1;
    hd.cap = s.c.logit_softcap;
    hd.p[0] = part_of(s.top, "head", s.c.logit_softcap > 0.f ? AXQ_ACT_SOFTCAP : AXQ_ACT_NONE, m->logits, s.c.vocab_size);
    hd.p[0].nw = vec(s.top, "final.norm");
    return axq_dense_gemv(ctx, norm_mode(s), norm_in(s, s.top, "final.norm", m->h), hd);
}

int axq_stack_rows(axq_model *m, const int32_t *toks, int nb, int pos0) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    const int W = s.c.width, ldw = pad64(W);
    const size_t es = s.f32 ? 4 : 2;
    const bool first = pos0 == 0, average = s.c.depth_average && !s.runs.empty();
    int rc;
    if ((rc = reserve_rows(m, nb))) return rc;
    const size_t stride = (size_t)nb * W;
    float *x = average ? s.r_past : s.r_h;
    if ((rc = axq_rows_embed(ctx, m->emb, m->emb32, vec(s.top, "pos"), toks, nullptr, pos0, nb, W, x))) return rc;
    for (size_t run = 0; run < s.runs.size(); run++) {
        Run &r = s.runs[run];
        Layer &l = s.layers[r.layer];
        const axq_layer_config &c = l.c;
        float *y = average ? s.r_past + (run + 1) * stride : s.r_h;
        const axq_avg avg = avg_of(s, l, s.r_past, stride, run, s.r_h);
        const bool parallel = s.c.parallel && c.ff > 0, mix = c.mixer == AXQ_MIX_WKV;
        axq_in in = norm_in(s, l, "norm1", x);
        in.prev = r.prev;
        Proj p;
        add_firsts(p, l, mixer_firsts(c), s.r_proj, nb, in.nw);
        const float *mu[AXQ_MAX_PARTS] = {};
        for (int i = 0; i < p.parts.n_parts; i++) {
            mu[i] = p.parts.p[i].mu;
            p.parts.p[i].x = reinterpret_cast<const uint8_t *>(s.r_x) + (mix ? (size_t)i * nb * ldw * es : 0);
        }
        const int mixers = p.parts.n_parts;
        float *const *ff = nullptr;
        if (parallel) {
            p.out.reserve(p.out.size() + 8);
            ff = p.out.data() + p.out.size();
            add_firsts(p, l, ff_firsts(c), s.r_z, nb, nullptr);
            for (int i = mixers; i < p.parts.n_parts; i++) p.parts.p[i].x = s.r_x2;
            ff_operands(s, c, p, mixers);
            if ((rc = axq_rows_layer_norm(ctx, in, nb, in.nw, {s.r_x, ldw, s.f32}, vec(l, "norm2"), {s.r_x2, ldw, s.f32}))) return rc;
        } else if (mix) {
            if ((rc = axq_rows_tanh_norm(ctx, in, nb, first, p.parts.n_parts, mu, {s.r_x, ldw, s.f32}))) return rc;
        } else if ((rc = norm_rows(ctx, s, in, nb, {s.r_x, ldw, s.f32}))) {
            return rc;
        }
        if ((rc = axq_dense_gemm(ctx, p.parts, nb, W, ldw, s.f32))) return rc;
        const int mo = mixer_out(c), ldo = pad64(mo);
        const axq_rows_out xo = {s.r_x, ldo, s.f32};
        if (c.mixer == AXQ_MIX_ATTENTION) {
            const axq_sig_attn a = attn_of(s, l, r, m->cfg.max_position_embeddings);
            if ((rc = axq_sig_attn_rows(ctx, a, p.out[0], p.out[1], p.out[2], p.width(0), p.width(1), p.width(2), nb, pos0, s.r_qs, xo))) return rc;
        } else if (c.mixer == AXQ_MIX_SOFTMAX) {
            const axq_soft_attn a = soft_attn_of(s, l, r, m->cfg.max_position_embeddings);
            const SoftIn i = soft_in(c, p);
            if ((rc = axq_soft_attn_rows(ctx, a, i.q, i.k, i.v, i.ldq, i.ldk, i.ldv, i.gate, nb, pos0, s.r_qs, xo))) return rc;
        } else {
            axq_linstate a = linstate_of(l, r, p, s.r_o);
            axq_in gate;
            gate.x = s.r_o;
            gate.k = mo;
            gate.eps = s.c.norm_eps;
            gate.nw = vec(l, "mix.norm");
            gate.gate = p.out[3];
            if (mix) { // the decay factors: a second, narrow product on the first one's tanh, in 32-bit
                float *decay = p.out[5];
                const int ld = c.heads * c.dim;
                if ((rc = axq_rows_zero_tail(ctx, nb, c.decay_rank, {p.out[4], p.width(4), true}))) return rc;
                axq_parts d = {};
                d.n_parts = 1;
                d.p[0] = part_of(l, "mix.w2", AXQ_ACT_DECAY, decay, ld);
                d.p[0].bias = vec(l, "mix.w0");
                d.p[0].x = p.out[4];
                if ((rc = axq_dense_gemm(ctx, d, nb, c.decay_rank, p.width(4), true))) return rc;
                a.wt = decay;
                a.ldw = ld;
                if ((rc = axq_store_prev(ctx, in, nb, r.prev))) return rc;
            }
            a.seg_state = s.r_seg;
            a.seg_decay = s.r_segw;
            if ((rc = axq_linstate_rows(ctx, a, nb, first))) return rc;
            if ((rc = axq_rows_rms_gate(ctx, gate, nb, mix ? c.dim : mo, xo))) return rc;
        }
        axq_parts o = {};
        o.n_parts = 1;
        o.p[0] = part_of(l, "mix.o", AXQ_ACT_NONE, y, W, x);
        o.p[0].x = s.r_x;
        if (c.ff <= 0) o.p[0].avg = avg;
        if ((rc = axq_dense_gemm(ctx, o, nb, mo, ldo, s.f32))) return rc;
        if (c.ff > 0) {
            Proj f;
            if (!parallel) {
                if ((rc = norm_rows(ctx, s, norm_in(s, l, "norm2", y), nb, {s.r_x, ldw, s.f32}))) return rc;
                add_firsts(f, l, ff_firsts(c), s.r_z, nb, nullptr);
                ff = f.out.data();
                for (int i = 0; i < f.parts.n_parts; i++) f.parts.p[i].x = s.r_x;
                ff_operands(s, c, f, 0);
                if ((rc = axq_dense_gemm(ctx, f.parts, nb, W, ldw, s.f32))) return rc;
            }
            if ((rc = ff_rows(ctx, s, l, ff, parallel ? s.r_x2 : s.r_x, nb, y, avg))) return rc;
        }
        x = s.r_h;
        if (s.trace)
            AXQ_HIP(ctx, hipMemcpyAsync(s.trace + ((size_t)run * s.trace_total + s.trace_row0) * W, s.r_h, (size_t)nb * W * 4, hipMemcpyDeviceToHost,
                                        ctx->stream), AXQ_ERR_COPY_FAILED);
    }
    s.trace = nullptr;
    AXQ_HIP(ctx, hipMemcpyAsync(m->h, s.r_h + (size_t)(nb - 1) * W, (size_t)W * 4, hipMemcpyDeviceToDevice, ctx->stream), AXQ_ERR_COPY_FAILED);
    return AXQ_OK;
}

int axq_stack_logits_rows(axq_model *m, const int32_t *rows, int n, float *logits) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    const int W = s.c.width, ldw = pad64(W), V = s.c.vocab_size;
    int rc;
    const int want = n < LOGITS_ROWS ? n : LOGITS_ROWS;
    if (want > s.logits_cap) {
        AXQ_HIP(ctx, hipStreamSynchronize(ctx->stream), AXQ_ERR_DRIVER);
        if (s.r_logits) (void)hipFree(s.r_logits);
        s.r_logits = nullptr;
        s.logits_cap = 0;
        AXQ_HIP(ctx, dev_alloc(&s.r_logits, (size_t)want * V * 4), AXQ_ERR_ALLOCATION_FAILED);
        if (!s.r_want) AXQ_HIP(ctx, dev_alloc(&s.r_want, LOGITS_ROWS * 4), AXQ_ERR_ALLOCATION_FAILED);
        s.logits_cap = want;
    }
    for (int j0 = 0; j0 < n; j0 += want) {
        const int nj = n - j0 < want ? n - j0 : want;
        AXQ_HIP(ctx, hipMemcpyAsync(s.r_want, rows + j0, (size_t)nj * 4, hipMemcpyHostToDevice, ctx->stream), AXQ_ERR_COPY_FAILED);
        axq_in in = norm_in(s, s.top, "final.norm", s.r_h);
        in.rows = s.r_want;
        if ((rc = norm_rows(ctx, s, in, nj, {s.r_x, ldw, s.f32}))) return rc;
        axq_parts hd = {};
        hd.n_parts = 1;
        hd.cap = s.c.logit_softcap;
        hd.p[0] = part_of(s.top, "head", s.c.logit_softcap > 0.f ? AXQ_ACT_SOFTCAP : AXQ_ACT_NONE, s.r_logits, V);
        hd.p[0].x = s.r_x;
        if ((rc = axq_dense_gemm(ctx, hd, nj, W, ldw, s.f32))) return rc;
        AXQ_HIP(ctx, hipMemcpyAsync(logits + (size_t)j0 * V, s.r_logits, (size_t)nj * V * 4, hipMemcpyDeviceToHost, ctx->stream), AXQ_ERR_COPY_FAILED);
    }
    return AXQ_OK;
}

void axq_stack_free(axq_model *m) {
    axq_stack *s = m->stack;
    if (!s) return;
    auto drop = [&](Layer &l) {
        for (auto &kv : l.t) {
            axq_weight_free(m->ctx, kv.second.w);
            if (kv.second.v) (void)hipFree(kv.second.v);
        }
        for (auto &kv : l.fused) axq_weight_free(m->ctx, kv.second);
        if (l.bias) (void)hipFree(l.bias);
        if (l.temp) (void)hipFree(l.temp);
    };
    for (Layer &l : s->layers) drop(l);
    drop(s->top);
    for (Run &r : s->runs)
        for (void *p : {r.kc, r.vc, r.pkc, r.pvc, (void *)r.state, (void *)r.prev})
            if (p) (void)hipFree(p);
    for (Rotation &r : s->rotations)
        for (void *p : {(void *)r.rc, (void *)r.rs})
            if (p) (void)hipFree(p);
    for (void *p : {(void *)s->proj, (void *)s->o, (void *)s->z, (void *)s->part, s->qs, (void *)s->r_h, (void *)s->r_proj, (void *)s->r_o,
                    (void *)s->r_z, (void *)s->r_logits, (void *)s->r_seg, (void *)s->r_segw, (void *)s->r_want, s->r_x, s->r_qs,
                    s->r_x2, s->r_f, (void *)s->r_past, s->r_ez, (void *)s->r_ey, (void *)s->r_wt, (void *)s->r_route, (void *)s->past,
                    (void *)s->ez, (void *)s->wt, (void *)s->sel})
        if (p) (void)hipFree(p);
    delete s;
    m->stack = nullptr;
}

namespace {

// A linear that has been made goes where its slot says.
int keep_linear(axq_model *m, Slot &t, axq_weight *w) {
    axq_ctx *ctx = m->ctx;
    hipError_t e = hipSuccess;
    if (t.into) {
        const size_t pitch = w->codes_pitch, group = AXQ_GLU_GROUP * pitch;
        uint8_t *dst = t.into->codes + (size_t)t.row0 * pitch;
        const int64_t whole = t.spread ? t.rows / AXQ_GLU_GROUP : 0, rest = t.rows - whole * AXQ_GLU_GROUP;
        if (whole) e = hipMemcpy2DAsync(dst, 2 * group, w->codes, group, group, (size_t)whole, hipMemcpyDeviceToDevice, ctx->stream);
        if (e == hipSuccess && rest)
            e = hipMemcpyAsync(dst + (size_t)whole * 2 * group, w->codes + (size_t)whole * group, (size_t)rest * pitch, hipMemcpyDeviceToDevice, ctx->stream);
    }
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    if (t.into || e != hipSuccess) {
        axq_weight_free(ctx, w);
    } else {
        axq_weight_free(ctx, t.w);
        t.w = w;
        axq_model_drop_graphs(m);
    }
    if (e != hipSuccess) return axq_fail(ctx, AXQ_ERR_COPY_FAILED, "a linear's rows: %s", hipGetErrorString(e));
    t.set = true;
    return AXQ_OK;
}

// A slot whose linear is rows row0 .. of `into`.
void add_slice(Layer &l, const std::string &name, int64_t rows, int64_t cols, axq_weight *into, int64_t row0, bool spread) {
    add_slot(l, name.c_str(), true, rows, cols);
    Slot &t = l.t[name];
    t.into = into;
    t.row0 = row0;
    t.spread = spread;
}

int add_fused(axq_ctx *ctx, Layer &l, const char *name, int64_t rows, int64_t cols, axq_weight **out) {
    axq_weight *w = nullptr;
    const int rc = axq_weight_alloc(ctx, AXQ_BF16, rows, cols, &w);
    if (rc) return rc;
    l.fused[name] = *out = w;
    AXQ_HIP(ctx, hipMemsetAsync(w->codes, 0, w->codes_pitch * (size_t)rows, ctx->stream), AXQ_ERR_DRIVER); // rows nobody sets are zeros
    return AXQ_OK;
}

int add_ff(axq_ctx *ctx, Layer &l, int W) {
    const axq_layer_config &c = l.c;
    int rc;
    axq_weight *up, *down;
    if (c.ff_kind == AXQ_FF_GLU) {
        if ((rc = add_fused(ctx, l, "mlp.gu", glu_rows(c.ff), W, &up))) return rc;
        add_slice(l, "mlp.gate", c.ff, W, up, 0, true);
        add_slice(l, "mlp.up", c.ff, W, up, AXQ_GLU_GROUP, true);
        add_slot(l, "mlp.down", true, W, c.ff);
    } else if (c.ff_kind == AXQ_FF_MOE) {
        if ((rc = add_fused(ctx, l, "mlp.experts.up", (int64_t)c.experts * c.ff, W, &up))) return rc;
        if ((rc = add_fused(ctx, l, "mlp.experts.down", (int64_t)c.experts * W, c.ff, &down))) return rc;
        for (int e = 0; e < c.experts; e++) {
            const std::string name = "mlp.e" + std::to_string(e);
            add_slice(l, name + ".up", c.ff, W, up, (int64_t)e * c.ff, false);
            add_slice(l, name + ".down", W, c.ff, down, (int64_t)e * W, false);
        }
        add_slot(l, "mlp.router", true, c.experts, W);
        if (c.shared_ff > 0) {
            add_slot(l, "mlp.shared.up", true, c.shared_ff, W);
            add_slot(l, "mlp.shared.down", true, W, c.shared_ff);
            add_slot(l, "mlp.shared.sg", true, 1, W);
        }
    } else {
        add_slot(l, "mlp.up", true, c.ff, W);
        add_slot(l, "mlp.down", true, W, c.ff);
        add_slot(l, "mlp.act", false, 1, 4);
    }
    return AXQ_OK;
}

// Angle of pair i at position p: p f_i, f_i = base^(-2 i / dims), slowed down by `factor` where a pair turns less than
// `slow` times over `original` positions, as it is where it turns more than `fast` times, a linear mix between (YaRN).
int add_rotation(axq_ctx *ctx, axq_stack &s, Layer &l, int cap) {
    const axq_layer_config &c = l.c;
    for (const Rotation &r : s.rotations)
        if (r.c.rot_dims == c.rot_dims && r.c.rot_base == c.rot_base && r.c.rot_original == c.rot_original && r.c.rot_factor == c.rot_factor &&
            r.c.rot_fast == c.rot_fast && r.c.rot_slow == c.rot_slow) {
            l.rc = r.rc;
            l.rs = r.rs;
            return AXQ_OK;
        }
    const int n = c.rot_dims / 2;
    std::vector<double> f(n);
    double size = 1.0, lo = 0.0, hi = 0.0;
    const bool yarn = c.rot_original > 0;
    if (yarn) {
        auto dim_of = [&](double turns) { return c.rot_dims * log(c.rot_original / (2.0 * M_PI * turns)) / (2.0 * log(c.rot_base)); };
        lo = fmax(floor(dim_of(c.rot_fast)), 0.0);
        hi = fmin(ceil(dim_of(c.rot_slow)), c.rot_dims - 1.0);
        size = 0.1 * log(c.rot_factor) + 1.0;
    }
    for (int i = 0; i < n; i++) {
        f[i] = pow(c.rot_base, -2.0 * i / c.rot_dims);
        if (yarn) {
            const double ramp = fmin(fmax((i - lo) / fmax(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / c.rot_factor * ramp + f[i] * (1.0 - ramp);
        }
    }
    std::vector<float> cs((size_t)cap * n), sn((size_t)cap * n);
    for (int p = 0; p < cap; p++)
        for (int i = 0; i < n; i++) {
            const double a = p * f[i];
            cs[(size_t)p * n + i] = (float)(cos(a) * size);
            sn[(size_t)p * n + i] = (float)(sin(a) * size);
        }
    s.rotations.emplace_back();
    Rotation &r = s.rotations.back();
    r.c = c;
    AXQ_HIP(ctx, dev_alloc(&r.rc, cs.size() * 4), AXQ_ERR_ALLOCATION_FAILED);
    AXQ_HIP(ctx, dev_alloc(&r.rs, sn.size() * 4), AXQ_ERR_ALLOCATION_FAILED);
    AXQ_HIP(ctx, hipMemcpy(r.rc, cs.data(), cs.size() * 4, hipMemcpyHostToDevice), AXQ_ERR_COPY_FAILED);
    AXQ_HIP(ctx, hipMemcpy(r.rs, sn.data(), sn.size() * 4, hipMemcpyHostToDevice), AXQ_ERR_COPY_FAILED);
    l.rc = r.rc;
    l.rs = r.rs;
    return AXQ_OK;
}

// Why a softmax attention layer cannot be made, or NULL.
const char *check_softmax(const axq_layer_config &l) {
    if (l.kv_heads < 1 || l.heads % l.kv_heads || l.vdim < 1 || l.vdim > 256) return "attention";
    if (l.window < 0 || l.pool < 0 || !(l.scale > 0.f)) return "window, pool or scale";
    if (l.keys_as_values && l.vdim != l.dim) return "values that are the keys have their size";
    if (l.rot_dims < 0 || l.rot_dims > l.dim || l.rot_dims % 2) return "rot_dims";
    if (l.rot_dims > 0 && !(l.rot_base > 0.0)) return "rot_base";
    if (l.rot_dims > 0 && l.rot_original > 0 && (!(l.rot_factor > 0.0) || !(l.rot_fast > 0.0) || !(l.rot_slow > 0.0) || l.rot_base == 1.0)) return "rotation scaling";
    if (l.heads / l.kv_heads * ((l.dim <= 64 ? 64 : l.dim <= 128 ? 128 : 256) + 64) * 4 > 128 * 1024) return "query heads per KV head";
    return nullptr;
}

const char *check_ff(const axq_stack_config &c, const axq_layer_config &l, int mixer_out) {
    auto steps = [](int k) { return (k + 511) / 512; };
    int total = c.parallel ? steps(mixer_out) : 0; // of the last product's input in a decode step
    if (l.ff_kind == AXQ_FF_GLU) {
        total += steps(l.ff);
    } else if (l.ff_kind == AXQ_FF_MOE) {
        if (l.experts < 1 || l.experts > AXQ_MOE_MAX_EXPERTS || l.groups < 1 || l.experts % l.groups || l.groups_keep < 1 || l.groups_keep > l.groups || l.top < 1 ||
            l.top > l.groups_keep * (l.experts / l.groups) || l.shared_ff < 0)
            return "experts, groups or top";
        if (c.norm != AXQ_NORM_LAYER) return "a mixture of experts comes with layer norms";
        if (l.top > AXQ_MAX_SEG_ITEMS - 2) return "experts per token";
        total += l.top * steps(l.ff) + steps(l.shared_ff);
    } else if (l.ff_kind != AXQ_FF_POLY) {
        return "an unknown feed-forward";
    } else if (c.parallel) {
        return "this feed-forward does not run in parallel layers";
    }
    return total > AXQ_DENSE_MAX_K / 512 ? "the feed-forward's width" : nullptr;
}

} // namespace

int axq_stack_random_init(axq_model *m, float std, uint64_t seed) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    int rc = AXQ_OK;
    size_t most = (size_t)s.c.vocab_size * s.c.width;
    auto each = [&](auto fn) {
        for (auto &kv : s.top.t)
            if (!rc) rc = fn(-1, kv.first, kv.second);
        for (size_t i = 0; i < s.layers.size(); i++)
            for (auto &kv : s.layers[i].t)
                if (!rc) rc = fn((int)i, kv.first, kv.second);
    };
    each([&](int, const std::string &, Slot &t) { if (t.linear && (size_t)(t.rows * t.cols) > most) most = (size_t)(t.rows * t.cols); return AXQ_OK; });
    float *tmp = nullptr;
    AXQ_HIP(ctx, dev_alloc(&tmp, most * 4), AXQ_ERR_ALLOCATION_FAILED);
    const float pb = -logf((float)m->cfg.max_position_embeddings);
    axq_model_drop_graphs(m);
    each([&](int layer, const std::string &name, Slot &t) -> int {
        if (t.linear) {
            int e = axq_fill_normal_f32(ctx, tmp, (size_t)(t.rows * t.cols), 0.f, std, 0.f, 0.f, ++seed);
            axq_weight *w = nullptr;
            if (!e) e = axq_weight_quantize(ctx, AXQ_BF16, t.rows, t.cols, tmp, AXQ_MEM_DEVICE, &w);
            return e ? e : keep_linear(m, t, w);
        }
        std::vector<float> v((size_t)(t.rows * t.cols));
        for (size_t i = 0; i < v.size(); i++) {
            if (name == "mix.decay") v[i] = expf(-exp2f(-8.f * (float)(i + 1) / (float)v.size()));
            else if (name == "mix.w0") v[i] = -6.f + 5.f * (float)(i % 64) / 63.f;
            else if (name == "mix.pb") v[i] = pb;
            else if (name == "dwa") v[i] = i + 1 == v.size() ? 0.7f : 0.3f / (float)(v.size() - 1);
            else if (name == "mlp.act") v[i] = i < 3 ? 1.f / 3.f : 0.f;
            else if (name == "mix.rel" || name == "pos" || (name.size() > 2 && name.substr(name.size() - 2) == ".b")) v[i] = 0.f;
            else if (name == "mix.u" || name.substr(0, 7) == "mix.mu." || (name.size() > 6 && name.substr(name.size() - 6) == ".alpha")) v[i] = 0.5f;
            else v[i] = 1.f; // norm weights
        }
        return axq_model_set_tensor(m, layer, name.c_str(), v.data(), t.rows, t.cols);
    });
    if (!rc) rc = axq_fill_normal_f32(ctx, tmp, (size_t)s.c.vocab_size * s.c.width, 0.f, 1.f, 0.f, 0.f, ++seed);
    if (!rc) rc = axq_model_set_embedding_f32(m, tmp, AXQ_MEM_DEVICE);
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(tmp);
    return rc;
}

extern "C" {

int axq_model_create_stack(axq_ctx *ctx, const axq_stack_config *cfg, axq_model **out) {
    if (!ctx) return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_create_stack: NULL context");
    if (!cfg || !out || (cfg->num_layers > 0 && !cfg->layers)) return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_create_stack: NULL pointer");
    *out = NULL;
    const axq_stack_config &c = *cfg;
    if (c.vocab_size < 1 || c.width < 1 || c.max_positions < 1 || c.num_layers < 0 || c.cache_positions < 0 || c.width > AXQ_DENSE_MAX_K)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: model dimensions must be positive, the width at most %d", AXQ_DENSE_MAX_K);
    if (c.compute != AXQ_COMPUTE_BF16 && c.compute != AXQ_COMPUTE_F32)
        return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_create_stack: compute must be AXQ_COMPUTE_BF16 or AXQ_COMPUTE_F32");
    const bool loop = c.loop_times > 1;
    if (loop && (c.loop_start < 0 || c.loop_stop <= c.loop_start || c.loop_stop > c.num_layers))
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: loop over layers %d .. %d of %d", c.loop_start, c.loop_stop, c.num_layers);
    if (c.norm != AXQ_NORM_TANH && c.norm != AXQ_NORM_LAYER)
        return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_create_stack: unknown norm %d", c.norm);
    if ((c.parallel && c.norm != AXQ_NORM_LAYER) || (c.depth_average && loop))
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: parallel layers come with layer norms, a mean over the layers without a loop");
    for (int i = 0; i < c.num_layers; i++) {
        const axq_layer_config &l = c.layers[i];
        const char *bad = nullptr;
        if (l.heads < 1 || l.dim < 1 || l.dim > 256 || l.ff < 0 || l.ff > AXQ_DENSE_MAX_K) bad = "heads, dim (at most 256) or ff";
        else if (l.mixer == AXQ_MIX_ATTENTION) {
            if (l.kv_heads < 1 || l.heads % l.kv_heads || l.vdim < 1 || l.vdim > 256 || l.bias_rows < 0 || l.bias_rows == 1 || l.q_temp_every < 0) bad = "attention";
        } else if (l.mixer == AXQ_MIX_LIGHTNING) {
            if (l.vdim < 1) bad = "vdim";
        } else if (l.mixer == AXQ_MIX_WKV) {
            if (l.decay_rank < 1) bad = "decay_rank";
            else if (c.norm != AXQ_NORM_TANH) bad = "time mixing comes with tanh norms";
        } else if (l.mixer == AXQ_MIX_SOFTMAX) {
            bad = check_softmax(l);
        } else {
            bad = "an unknown mixer";
        }
        if (!bad && mixer_out(l) > AXQ_DENSE_MAX_K) bad = "heads times vdim";
        if (!bad && l.ff > 0) bad = check_ff(c, l, mixer_out(l));
        if (bad) return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: layer %d: %s", i, bad);
    }
    AXQ_HIP(ctx, hipSetDevice(ctx->device), AXQ_ERR_DRIVER);
    axq_model *m = new (std::nothrow) axq_model();
    if (!m) return axq_fail(ctx, AXQ_ERR_ALLOCATION_FAILED, "out of host memory");
    m->ctx = ctx;
    m->cfg.vocab_size = c.vocab_size;
    m->cfg.hidden_size = c.width;
    m->cfg.num_hidden_layers = c.num_layers;
    m->cfg.rms_norm_eps = c.norm_eps;
    const int cap = c.cache_positions > 0 && c.cache_positions < c.max_positions ? c.cache_positions : c.max_positions;
    m->cfg.max_position_embeddings = cap;
    m->stack = new (std::nothrow) axq_stack();
    int rc = m->stack ? axq_model_alloc_common(m) : axq_fail(ctx, AXQ_ERR_ALLOCATION_FAILED, "out of host memory");
    if (rc) {
        axq_model_free(m);
        return rc;
    }
    axq_stack &s = *m->stack;
    s.c = c;
    s.c.layers = nullptr; // the caller's array is not kept
    s.f32 = c.compute == AXQ_COMPUTE_F32;
    const int W = c.width;
    if (c.position_table) add_slot(s.top, "pos", false, c.max_positions, W);
    add_norm(s.top, "final.norm", W, c.norm);
    add_slot(s.top, "head", true, c.vocab_size, W);
    hipError_t e = hipSuccess;
#define TRY(x) if (e == hipSuccess) e = (x)
    size_t proj = 0, o = 0, z = 0, part = 0, qs = 0, ez = 0, top = 0;
    for (int i = 0; i < c.num_layers && !rc; i++) {
        s.layers.emplace_back();
        Layer &l = s.layers.back();
        l.c = c.layers[i];
        axq_layer_config &lc = l.c;
        add_norm(l, "norm1", W, c.norm);
        if (c.depth_average) add_slot(l, "dwa", false, 1, i + 2);
        const int64_t hd = (int64_t)lc.heads * lc.dim, mo = mixer_out(lc);
        if (lc.mixer == AXQ_MIX_ATTENTION) {
            add_slot(l, "mix.q", true, hd, W);
            add_slot(l, "mix.k", true, (int64_t)lc.kv_heads * lc.dim, W);
            add_slot(l, "mix.v", true, (int64_t)lc.kv_heads * lc.vdim, W);
            add_slot(l, "mix.q.norm", false, 1, lc.dim);
            add_slot(l, "mix.k.norm", false, 1, lc.dim);
            if (lc.bias_rows > 0) add_slot(l, "mix.rel", false, lc.bias_rows, lc.heads);
            add_slot(l, "mix.pb", false, 1, lc.heads);
            std::vector<float> temp(cap, 1.0f);
            if (lc.q_temp_every > 0)
                for (int p = 0; p < cap; p++) temp[p] = (float)(1.0 + (double)lc.q_temp_coef * log((double)((p + 1) / lc.q_temp_every) + 1.0));
            TRY(dev_alloc(&l.temp, (size_t)cap * 4));
            TRY(hipMemcpy(l.temp, temp.data(), (size_t)cap * 4, hipMemcpyHostToDevice));
            axq_sig_attn a = {};
            a.heads = lc.heads; a.kv_heads = lc.kv_heads; a.dim = lc.dim; a.vdim = lc.vdim; a.cap = cap; a.f32 = s.f32;
            const size_t pb = axq_sig_attn_part_bytes(a), qb = axq_sig_attn_q_bytes(a, 1);
            part = pb > part ? pb : part;
            qs = qb > qs ? qb : qs;
        } else if (lc.mixer == AXQ_MIX_SOFTMAX) {
            add_slot(l, "mix.q", true, hd, W);
            add_slot(l, "mix.k", true, (int64_t)lc.kv_heads * lc.dim, W);
            if (!lc.keys_as_values) add_slot(l, "mix.v", true, (int64_t)lc.kv_heads * lc.vdim, W);
            if (lc.head_gate) add_slot(l, "mix.g", true, lc.heads, W);
            if (lc.rot_dims > 0 && e == hipSuccess) rc = add_rotation(ctx, s, l, cap);
            const axq_soft_attn a = soft_attn_of(s, l, Run(), cap);
            const size_t pb = axq_soft_attn_part_bytes(a), qb = axq_soft_attn_q_bytes(a, 1);
            part = pb > part ? pb : part;
            qs = qb > qs ? qb : qs;
        } else if (lc.mixer == AXQ_MIX_LIGHTNING) {
            add_slot(l, "mix.q", true, hd, W);
            add_slot(l, "mix.k", true, hd, W);
            add_slot(l, "mix.v", true, mo, W);
            add_slot(l, "mix.g", true, mo, W);
            add_slot(l, "mix.norm", false, 1, mo);
            add_slot(l, "mix.decay", false, 1, lc.heads);
        } else {
            for (const char *n : {"mix.r", "mix.k", "mix.v", "mix.g"}) add_slot(l, n, true, hd, W);
            for (const char *n : {"mix.mu.r", "mix.mu.k", "mix.mu.v", "mix.mu.g", "mix.mu.w"}) add_slot(l, n, false, 1, W);
            add_slot(l, "mix.w1", true, lc.decay_rank, W);
            add_slot(l, "mix.w2", true, hd, lc.decay_rank);
            add_slot(l, "mix.w0", false, 1, hd);
            add_slot(l, "mix.u", false, lc.heads, lc.dim);
            add_slot(l, "mix.norm", false, 1, hd);
        }
        add_slot(l, "mix.o", true, W, mo);
        if (lc.ff > 0) {
            add_norm(l, "norm2", W, c.norm);
            if (!rc) rc = add_ff(ctx, l, W);
            const size_t n = total_width(ff_firsts(lc)), t = lc.ff_kind == AXQ_FF_MOE ? lc.top : 0;
            z = n > z ? n : z;
            ez = t * lc.ff > ez ? t * lc.ff : ez;
            top = t > top ? t : top;
        }
        const size_t n = proj_width(lc);
        proj = n > proj ? n : proj;
        o = (size_t)mo > o ? mo : o;
    }
    if (rc) {
        axq_model_free(m);
        return rc;
    }
    std::vector<int> order;
    if (!loop) {
        for (int i = 0; i < c.num_layers; i++) order.push_back(i);
    } else {
        for (int i = 0; i < c.loop_start; i++) order.push_back(i);
        for (int t = 0; t < c.loop_times; t++)
            for (int i = c.loop_start; i < c.loop_stop; i++) order.push_back(i);
        for (int i = c.loop_stop; i < c.num_layers; i++) order.push_back(i);
    }
    for (int i : order) {
        s.runs.emplace_back();
        Run &r = s.runs.back();
        r.layer = i;
        const axq_layer_config &lc = s.layers[i].c;
        if (lc.mixer == AXQ_MIX_ATTENTION) {
            axq_sig_attn a = {};
            a.kv_heads = lc.kv_heads; a.dim = lc.dim; a.vdim = lc.vdim; a.cap = cap; a.f32 = s.f32;
            const size_t kb = axq_sig_attn_k_bytes(a), vb = axq_sig_attn_v_bytes(a);
            TRY(dev_alloc((uint8_t **)&r.kc, kb));
            TRY(dev_alloc((uint8_t **)&r.vc, vb));
            TRY(hipMemsetAsync(r.kc, 0, kb, ctx->stream)); // the f16 cache's padding is multiplied with zeros, so it must be finite
            TRY(hipMemsetAsync(r.vc, 0, vb, ctx->stream));
        } else if (lc.mixer == AXQ_MIX_SOFTMAX) {
            const axq_soft_attn a = soft_attn_of(s, s.layers[i], r, cap);
            const struct { void **p; size_t bytes; } caches[] = {{&r.kc, axq_soft_attn_k_bytes(a)}, {&r.vc, axq_soft_attn_v_bytes(a)},
                                                                 {&r.pkc, axq_soft_attn_pk_bytes(a)}, {&r.pvc, axq_soft_attn_pv_bytes(a)}};
            for (const auto &k : caches) {
                TRY(dev_alloc(k.p, k.bytes));
                if (k.bytes) TRY(hipMemsetAsync(*k.p, 0, k.bytes, ctx->stream)); // (see above)
            }
        } else {
            TRY(dev_alloc(&r.state, (size_t)lc.heads * lc.dim * (lc.mixer == AXQ_MIX_WKV ? lc.dim : lc.vdim) * 4));
            if (lc.mixer == AXQ_MIX_WKV) TRY(dev_alloc(&r.prev, (size_t)W * 4));
        }
    }
    TRY(dev_alloc(&s.proj, proj * 4));
    TRY(dev_alloc(&s.o, o * 4));
    TRY(dev_alloc(&s.z, z * 4));
    TRY(dev_alloc(&s.ez, ez * 4));
    TRY(dev_alloc(&s.wt, top * 4));
    TRY(dev_alloc(&s.sel, top * 4));
    if (c.depth_average) TRY(dev_alloc(&s.past, (s.runs.size() + 1) * (size_t)W * 4));
    TRY(dev_alloc(&s.part, part));
    TRY(dev_alloc((uint8_t **)&s.qs, qs));
    TRY(hipStreamSynchronize(ctx->stream));
#undef TRY
    if (e != hipSuccess) {
        rc = axq_fail(ctx, AXQ_ERR_ALLOCATION_FAILED, "model buffers: %s", hipGetErrorString(e));
        axq_model_free(m);
        return rc;
    }
    *out = m;
    return AXQ_OK;
}

int axq_model_set_tensor(axq_model *m, int layer, const char *name, const float *data, int64_t rows, int64_t cols) {
    if (!m || !name || !data) return AXQ_ERR_INVALID_ARGUMENT;
    axq_ctx *ctx = m->ctx;
    if (!m->stack) return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_set_tensor: the model has no described layers");
    axq_stack &s = *m->stack;
    if (layer < -1 || layer >= (int)s.layers.size()) return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_set_tensor: layer %d out of range", layer);
    Layer &l = layer < 0 ? s.top : s.layers[layer];
    auto it = l.t.find(name);
    if (it == l.t.end()) return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_model_set_tensor: layer %d has no tensor '%s'", layer, name);
    Slot &t = it->second;
    if (rows != t.rows || cols != t.cols)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: %s of layer %d: expected [%lld, %lld], got [%lld, %lld]", name, layer,
                        (long long)t.rows, (long long)t.cols, (long long)rows, (long long)cols);
    AXQ_HIP(ctx, hipSetDevice(ctx->device), AXQ_ERR_DRIVER);
    const size_t n = (size_t)(rows * cols);
    if (t.linear) {
        if (s.f32) // weights are kept in bfloat16: in 32-bit they must be such numbers
            for (size_t i = 0; i < n; i++) {
                uint32_t u;
                memcpy(&u, data + i, 4);
                if (u & 0xFFFFu) return axq_fail(ctx, AXQ_ERR_INVALID_DATA, "Invalid quantized data: %s of layer %d does not fit bfloat16 exactly", name, layer);
            }
        axq_weight *w = nullptr;
        int rc = axq_weight_quantize(ctx, AXQ_BF16, rows, cols, data, AXQ_MEM_HOST, &w);
        if (rc) return rc;
        return keep_linear(m, t, w);
    } else {
        AXQ_HIP(ctx, hipStreamSynchronize(ctx->stream), AXQ_ERR_DRIVER);
        if (!t.v) AXQ_HIP(ctx, dev_alloc(&t.v, n * 4), AXQ_ERR_ALLOCATION_FAILED);
        AXQ_HIP(ctx, hipMemcpy(t.v, data, n * 4, hipMemcpyHostToDevice), AXQ_ERR_COPY_FAILED);
        const bool keep = strcmp(name, "mix.rel") == 0 || strcmp(name, "mix.pb") == 0;
        if (keep) {
            t.host.assign(data, data + n);
            l.bias_ready = false;
        }
    }
    t.set = true;
    return AXQ_OK;
}

} // extern "C"
