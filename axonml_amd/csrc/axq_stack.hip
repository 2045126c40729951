// Models of described layers: a list of layer descriptions (mixer, sizes, feed-forward) run in order, a range of them
// possibly several times, each pass with its own cache or state.  The model is an axq_model: its tokens, positions,
// history, sampling, graphs and generation are those of axq_decode.hip, which calls the step and the rows here.
//
// A decode step is three kernels per recurrent layer (projections with the norm in front and the activations behind;
// state update; output projection with the gated norm in front and the residual add behind) and four plus two for
// attention with a feed-forward.  A prompt's rows take the same mechanisms in their row form: a norm or gate pass that
// writes the product's operand, one product launch for all projections that read it, the recurrence or attention.
// The residual stream, norms, scores, states and everything that enters a recurrence beyond the projections are f32.
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
};

struct Layer {
    axq_layer_config c;
    std::map<std::string, Slot> t;
    float *bias = nullptr; // attention: [heads][nt]
    int nt = 1;
    bool bias_ready = false;
    float *temp = nullptr; // attention: [cache positions]
};

struct Run {
    int layer;
    void *kc = nullptr, *vc = nullptr;
    float *state = nullptr, *prev = nullptr;
};

} // namespace

struct axq_stack {
    axq_stack_config c;
    bool f32;
    std::vector<Layer> layers;
    Layer top; // pos, final.norm, head
    std::vector<Run> runs;
    // activations of a step
    float *proj = nullptr, *o = nullptr, *z = nullptr, *part = nullptr;
    void *qs = nullptr;
    // activations of `cap` rows
    int cap = 0;
    float *r_h = nullptr, *r_proj = nullptr, *r_o = nullptr, *r_z = nullptr, *r_logits = nullptr;
    float *r_seg = nullptr, *r_segw = nullptr; // segments of a recurrence
    void *r_x = nullptr, *r_qs = nullptr;
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

void add_norm(Layer &l, const std::string &name, int64_t width) {
    add_slot(l, name.c_str(), false, 1, width);
    add_slot(l, (name + ".b").c_str(), false, 1, width);
    add_slot(l, (name + ".alpha").c_str(), false, 1, 1);
}

int mixer_out(const axq_layer_config &c) { return c.heads * (c.mixer == AXQ_MIX_WKV ? c.dim : c.vdim); }

// widths of a layer's first products, in launch order
std::vector<int> proj_widths(const axq_layer_config &c) {
    switch (c.mixer) {
    case AXQ_MIX_ATTENTION: return {c.heads * c.dim, c.kv_heads * c.dim, c.kv_heads * c.vdim};
    case AXQ_MIX_LIGHTNING: return {c.heads * c.dim, c.heads * c.dim, c.heads * c.vdim, c.heads * c.vdim};
    default: return {c.heads * c.dim, c.heads * c.dim, c.heads * c.dim, c.heads * c.dim, pad64(c.decay_rank), c.heads * c.dim}; // r k v g w1, then the decay
    }
}

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

float *vec(Layer &l, const char *name) { return l.t[name].v; }

axq_in norm_in(const axq_stack &s, Layer &l, const std::string &name, const float *x) {
    axq_in in;
    in.x = x;
    in.k = s.c.width;
    in.eps = s.c.norm_eps;
    in.alpha = vec(l, (name + ".alpha").c_str());
    in.nw = vec(l, name.c_str());
    in.nb = vec(l, (name + ".b").c_str());
    return in;
}

axq_part part_of(Layer &l, const char *name, int act, float *y, int ldy, bool add = false) {
    const axq_weight *w = l.t[name].w;
    axq_part p = {};
    p.w = reinterpret_cast<const uint16_t *>(w->codes);
    p.ldw = (int)(w->codes_pitch / 2);
    p.n = (int)w->n_rows;
    p.act = act;
    p.add = add ? 1 : 0;
    p.y = y;
    p.ldy = ldy;
    return p;
}

// The first products of a layer over `m` rows; part i's results are a block [m][widths[i]] of proj (out[i]).
struct Proj {
    axq_parts parts = {};
    std::vector<int> widths;
    std::vector<float *> out;
};

Proj make_proj(Layer &l, float *proj, int m) {
    Proj p;
    p.widths = proj_widths(l.c);
    for (int w : p.widths) {
        p.out.push_back(proj);
        proj += (size_t)w * m;
    }
    static const struct { const char *name; int act; const char *mu; } att[] = {{"mix.q", AXQ_ACT_NONE, nullptr}, {"mix.k", AXQ_ACT_NONE, nullptr}, {"mix.v", AXQ_ACT_NONE, nullptr}},
        lig[] = {{"mix.q", AXQ_ACT_SILU, nullptr}, {"mix.k", AXQ_ACT_SILU, nullptr}, {"mix.v", AXQ_ACT_SILU, nullptr}, {"mix.g", AXQ_ACT_SIGMOID, nullptr}},
        wkv[] = {{"mix.r", AXQ_ACT_NONE, "mix.mu.r"}, {"mix.k", AXQ_ACT_NONE, "mix.mu.k"}, {"mix.v", AXQ_ACT_NONE, "mix.mu.v"}, {"mix.g", AXQ_ACT_SILU, "mix.mu.g"}, {"mix.w1", AXQ_ACT_TANH, "mix.mu.w"}};
    const auto *list = l.c.mixer == AXQ_MIX_ATTENTION ? att : (l.c.mixer == AXQ_MIX_LIGHTNING ? lig : wkv);
    p.parts.n_parts = l.c.mixer == AXQ_MIX_ATTENTION ? 3 : (l.c.mixer == AXQ_MIX_LIGHTNING ? 4 : 5);
    for (int i = 0; i < p.parts.n_parts; i++) {
        p.parts.p[i] = part_of(l, list[i].name, list[i].act, p.out[i], p.widths[i]);
        if (list[i].mu) p.parts.p[i].mu = vec(l, list[i].mu);
    }
    return p;
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

axq_linstate linstate_of(Layer &l, const Run &r, const Proj &p, float *o) {
    axq_linstate a = {};
    const axq_layer_config &c = l.c;
    a.heads = c.heads;
    a.dk = c.dim;
    a.dv = c.mixer == AXQ_MIX_WKV ? c.dim : c.vdim;
    a.q = p.out[0]; a.k = p.out[1]; a.v = p.out[2];
    a.ldq = p.widths[0]; a.ldk = p.widths[1]; a.ldv = p.widths[2];
    if (c.mixer == AXQ_MIX_LIGHTNING) a.decay = vec(l, "mix.decay");
    else a.u = vec(l, "mix.u");
    a.state = r.state;
    a.o = o;
    return a;
}

int reserve_rows(axq_model *m, int rows) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    if (rows <= s.cap) return AXQ_OK;
    int cap = 64;
    while (cap < rows) cap *= 2;
    AXQ_HIP(ctx, hipStreamSynchronize(ctx->stream), AXQ_ERR_DRIVER);
    for (void **p : {(void **)&s.r_h, (void **)&s.r_proj, (void **)&s.r_o, (void **)&s.r_z, (void **)&s.r_seg, (void **)&s.r_segw, &s.r_x, &s.r_qs}) {
        if (*p) (void)hipFree(*p);
        *p = nullptr;
    }
    s.cap = 0;
    size_t proj = 0, o = 0, z = 0, x = pad64(s.c.width), qs = 0, seg = 0, segw = 0;
    for (Layer &l : s.layers) {
        size_t n = 0;
        for (int w : proj_widths(l.c)) n += w;
        proj = n > proj ? n : proj;
        const size_t mo = mixer_out(l.c);
        o = mo > o ? mo : o;
        z = (size_t)l.c.ff > z ? l.c.ff : z;
        size_t nx = pad64((int)mo);
        if (l.c.mixer == AXQ_MIX_WKV) nx = nx > (size_t)5 * pad64(s.c.width) ? nx : (size_t)5 * pad64(s.c.width);
        if (l.c.ff > 0 && nx < (size_t)pad64(l.c.ff)) nx = pad64(l.c.ff);
        x = nx > x ? nx : x;
        if (l.c.mixer == AXQ_MIX_ATTENTION) {
            axq_sig_attn a = {};
            a.heads = l.c.heads; a.dim = l.c.dim; a.f32 = s.f32;
            const size_t b = axq_sig_attn_q_bytes(a, 1);
            qs = b > qs ? b : qs;
        } else {
            const size_t w = (size_t)l.c.heads * l.c.dim, n = w * (l.c.mixer == AXQ_MIX_WKV ? l.c.dim : l.c.vdim);
            seg = n > seg ? n : seg;
            segw = w > segw ? w : segw;
        }
    }
    hipError_t e = dev_alloc(&s.r_h, (size_t)cap * s.c.width * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_proj, (size_t)cap * proj * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_o, (size_t)cap * o * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_z, (size_t)cap * z * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_x, (size_t)cap * x * (s.f32 ? 4 : 2));
    if (e == hipSuccess) e = dev_alloc(&s.r_qs, (size_t)cap * qs);
    if (e == hipSuccess) e = dev_alloc(&s.r_seg, seg * AXQ_LINSTATE_SEGS * 4);
    if (e == hipSuccess) e = dev_alloc(&s.r_segw, segw * AXQ_LINSTATE_SEGS * 4);
    if (e != hipSuccess) return axq_fail(ctx, AXQ_ERR_ALLOCATION_FAILED, "activations for %d rows: %s", cap, hipGetErrorString(e));
    s.cap = cap;
    return AXQ_OK;
}

} // namespace

int axq_stack_layer_runs(const axq_model *m) { return (int)m->stack->runs.size(); }

bool axq_stack_recurrent(const axq_model *m) {
    for (const Layer &l : m->stack->layers)
        if (l.c.mixer != AXQ_MIX_ATTENTION) return true;
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
    int rc;
    if ((rc = axq_rows_embed(ctx, m->emb, m->emb32, vec(s.top, "pos"), m->tok, m->pos, 0, 1, W, m->h))) return rc;
    for (Run &r : s.runs) {
        Layer &l = s.layers[r.layer];
        const axq_layer_config &c = l.c;
        Proj p = make_proj(l, s.proj, 1);
        axq_in in = norm_in(s, l, "norm1", m->h), out_in;
        int out_mode = AXQ_IN_PLAIN;
        in.prev = r.prev;
        in.pos = m->pos;
        if ((rc = axq_dense_gemv(ctx, c.mixer == AXQ_MIX_WKV ? AXQ_IN_TANH_NORM_MIX : AXQ_IN_TANH_NORM, in, p.parts))) return rc;
        out_in.x = s.o;
        out_in.k = mixer_out(c);
        out_in.eps = s.c.norm_eps;
        if (c.mixer == AXQ_MIX_ATTENTION) {
            const axq_sig_attn a = attn_of(s, l, r, m->cfg.max_position_embeddings);
            if ((rc = axq_sig_attn_token(ctx, a, p.out[0], p.out[1], p.out[2], m->pos, s.qs, s.part, s.o))) return rc;
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
        axq_parts o = {};
        o.n_parts = 1;
        o.p[0] = part_of(l, "mix.o", AXQ_ACT_NONE, m->h, W, true);
        if ((rc = axq_dense_gemv(ctx, out_mode, out_in, o))) return rc;
        if (c.ff > 0) {
            axq_parts u = {};
            u.n_parts = 1;
            u.p[0] = part_of(l, "mlp.up", AXQ_ACT_NONE, s.z, c.ff);
            if ((rc = axq_dense_gemv(ctx, AXQ_IN_TANH_NORM, norm_in(s, l, "norm2", m->h), u))) return rc;
            axq_in zin;
            zin.x = s.z;
            zin.k = c.ff;
            zin.eps = s.c.norm_eps;
            zin.coef = vec(l, "mlp.act");
            u.p[0] = part_of(l, "mlp.down", AXQ_ACT_NONE, m->h, W, true);
            if ((rc = axq_dense_gemv(ctx, AXQ_IN_POLY_NORM, zin, u))) return rc;
        }
    }
    axq_parts hd = {};
    hd.n_parts = 1;
    hd.cap = s.c.logit_softcap;
    hd.p[0] = part_of(s.top, "head", s.c.logit_softcap > 0.f ? AXQ_ACT_SOFTCAP : AXQ_ACT_NONE, m->logits, s.c.vocab_size);
    return axq_dense_gemv(ctx, AXQ_IN_TANH_NORM, norm_in(s, s.top, "final.norm", m->h), hd);
}

int axq_stack_rows(axq_model *m, const int32_t *toks, int nb, int pos0) {
    axq_stack &s = *m->stack;
    axq_ctx *ctx = m->ctx;
    const int W = s.c.width, ldw = pad64(W);
    const size_t es = s.f32 ? 4 : 2;
    const bool first = pos0 == 0;
    int rc;
    if ((rc = reserve_rows(m, nb))) return rc;
    if ((rc = axq_rows_embed(ctx, m->emb, m->emb32, vec(s.top, "pos"), toks, nullptr, pos0, nb, W, s.r_h))) return rc;
    for (size_t run = 0; run < s.runs.size(); run++) {
        Run &r = s.runs[run];
        Layer &l = s.layers[r.layer];
        const axq_layer_config &c = l.c;
        Proj p = make_proj(l, s.r_proj, nb);
        axq_in in = norm_in(s, l, "norm1", s.r_h);
        in.prev = r.prev;
        const bool mix = c.mixer == AXQ_MIX_WKV;
        const float *mu[AXQ_MAX_PARTS] = {};
        for (int i = 0; i < p.parts.n_parts; i++) {
            mu[i] = p.parts.p[i].mu;
            p.parts.p[i].x = reinterpret_cast<const uint8_t *>(s.r_x) + (mix ? (size_t)i * nb * ldw * es : 0);
        }
        if ((rc = axq_rows_tanh_norm(ctx, in, nb, first, mix ? p.parts.n_parts : 0, mu, {s.r_x, ldw, s.f32}))) return rc;
        if ((rc = axq_dense_gemm(ctx, p.parts, nb, W, ldw, s.f32))) return rc;
        const int mo = mixer_out(c), ldo = pad64(mo);
        const axq_rows_out xo = {s.r_x, ldo, s.f32};
        if (c.mixer == AXQ_MIX_ATTENTION) {
            const axq_sig_attn a = attn_of(s, l, r, m->cfg.max_position_embeddings);
            if ((rc = axq_sig_attn_rows(ctx, a, p.out[0], p.out[1], p.out[2], p.widths[0], p.widths[1], p.widths[2], nb, pos0, s.r_qs, xo))) return rc;
        } else {
            axq_linstate a = linstate_of(l, r, p, s.r_o);
            axq_in gate;
            gate.x = s.r_o;
            gate.k = mo;
            gate.eps = s.c.norm_eps;
            gate.nw = vec(l, "mix.norm");
            gate.gate = p.out[3];
            if (mix) { // the decay factors: a second, narrow product on the first one's tanh, in 32-bit
                if ((rc = axq_rows_zero_tail(ctx, nb, c.decay_rank, {p.out[4], p.widths[4], true}))) return rc;
                axq_parts d = {};
                d.n_parts = 1;
                d.p[0] = part_of(l, "mix.w2", AXQ_ACT_DECAY, p.out[5], p.widths[5]);
                d.p[0].bias = vec(l, "mix.w0");
                d.p[0].x = p.out[4];
                if ((rc = axq_dense_gemm(ctx, d, nb, c.decay_rank, p.widths[4], true))) return rc;
                a.wt = p.out[5];
                a.ldw = p.widths[5];
                if ((rc = axq_store_prev(ctx, in, nb, r.prev))) return rc;
            }
            a.seg_state = s.r_seg;
            a.seg_decay = s.r_segw;
            if ((rc = axq_linstate_rows(ctx, a, nb, first))) return rc;
            if ((rc = axq_rows_rms_gate(ctx, gate, nb, mix ? c.dim : mo, xo))) return rc;
        }
        axq_parts o = {};
        o.n_parts = 1;
        o.p[0] = part_of(l, "mix.o", AXQ_ACT_NONE, s.r_h, W, true);
        o.p[0].x = s.r_x;
        if ((rc = axq_dense_gemm(ctx, o, nb, mo, ldo, s.f32))) return rc;
        if (c.ff > 0) {
            if ((rc = axq_rows_tanh_norm(ctx, norm_in(s, l, "norm2", s.r_h), nb, first, 0, nullptr, {s.r_x, ldw, s.f32}))) return rc;
            axq_parts u = {};
            u.n_parts = 1;
            u.p[0] = part_of(l, "mlp.up", AXQ_ACT_NONE, s.r_z, c.ff);
            u.p[0].x = s.r_x;
            if ((rc = axq_dense_gemm(ctx, u, nb, W, ldw, s.f32))) return rc;
            axq_in zin;
            zin.x = s.r_z;
            zin.k = c.ff;
            zin.eps = s.c.norm_eps;
            zin.coef = vec(l, "mlp.act");
            const int ldf = pad64(c.ff);
            if ((rc = axq_rows_poly_norm(ctx, zin, nb, {s.r_x, ldf, s.f32}))) return rc;
            u.p[0] = part_of(l, "mlp.down", AXQ_ACT_NONE, s.r_h, W, true);
            u.p[0].x = s.r_x;
            if ((rc = axq_dense_gemm(ctx, u, nb, c.ff, ldf, s.f32))) return rc;
        }
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
        if ((rc = axq_rows_tanh_norm(ctx, in, nj, true, 0, nullptr, {s.r_x, ldw, s.f32}))) return rc;
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
        if (l.bias) (void)hipFree(l.bias);
        if (l.temp) (void)hipFree(l.temp);
    };
    for (Layer &l : s->layers) drop(l);
    drop(s->top);
    for (Run &r : s->runs)
        for (void *p : {r.kc, r.vc, (void *)r.state, (void *)r.prev})
            if (p) (void)hipFree(p);
    for (void *p : {(void *)s->proj, (void *)s->o, (void *)s->z, (void *)s->part, s->qs, (void *)s->r_h, (void *)s->r_proj, (void *)s->r_o,
                    (void *)s->r_z, (void *)s->r_logits, (void *)s->r_seg, (void *)s->r_segw, (void *)s->r_want, s->r_x, s->r_qs})
        if (p) (void)hipFree(p);
    delete s;
    m->stack = nullptr;
}

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
            axq_weight_free(ctx, t.w);
            t.w = nullptr;
            if (!e) e = axq_weight_quantize(ctx, AXQ_BF16, t.rows, t.cols, tmp, AXQ_MEM_DEVICE, &t.w);
            t.set = !e;
            return e;
        }
        std::vector<float> v((size_t)(t.rows * t.cols));
        for (size_t i = 0; i < v.size(); i++) {
            if (name == "mix.decay") v[i] = expf(-exp2f(-8.f * (float)(i + 1) / (float)v.size()));
            else if (name == "mix.w0") v[i] = -6.f + 5.f * (float)(i % 64) / 63.f;
            else if (name == "mix.pb") v[i] = pb;
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
        } else {
            bad = "an unknown mixer";
        }
        if (!bad && mixer_out(l) > AXQ_DENSE_MAX_K) bad = "heads times vdim";
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
    add_slot(s.top, "pos", false, c.max_positions, W);
    add_norm(s.top, "final.norm", W);
    add_slot(s.top, "head", true, c.vocab_size, W);
    hipError_t e = hipSuccess;
#define TRY(x) if (e == hipSuccess) e = (x)
    size_t proj = 0, o = 0, z = 0, part = 0, qs = 0;
    for (int i = 0; i < c.num_layers; i++) {
        s.layers.emplace_back();
        Layer &l = s.layers.back();
        l.c = c.layers[i];
        axq_layer_config &lc = l.c;
        add_norm(l, "norm1", W);
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
            add_norm(l, "norm2", W);
            add_slot(l, "mlp.up", true, lc.ff, W);
            add_slot(l, "mlp.down", true, W, lc.ff);
            add_slot(l, "mlp.act", false, 1, 4);
        }
        size_t n = 0;
        for (int w : proj_widths(lc)) n += w;
        proj = n > proj ? n : proj;
        o = (size_t)mo > o ? mo : o;
        z = (size_t)lc.ff > z ? lc.ff : z;
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
        } else {
            TRY(dev_alloc(&r.state, (size_t)lc.heads * lc.dim * (lc.mixer == AXQ_MIX_WKV ? lc.dim : lc.vdim) * 4));
            if (lc.mixer == AXQ_MIX_WKV) TRY(dev_alloc(&r.prev, (size_t)W * 4));
        }
    }
    TRY(dev_alloc(&s.proj, proj * 4));
    TRY(dev_alloc(&s.o, o * 4));
    TRY(dev_alloc(&s.z, z * 4));
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
        AXQ_HIP(ctx, hipStreamSynchronize(ctx->stream), AXQ_ERR_DRIVER);
        axq_weight_free(ctx, t.w);
        t.w = w;
        axq_model_drop_graphs(m);
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
