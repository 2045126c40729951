// Products with bfloat16 weights and the layers' row operations around them (internal).
//
// A product takes up to AXQ_MAX_PARTS weights that read the same width: one launch serves the projections of a layer.
// Weights are AXQ_BF16 (rows padded with zeros to a multiple of 64 elements), accumulation is in f32 everywhere.
#pragma once
#include "axq_internal.h"

#define AXQ_MAX_PARTS 8

// What happens to a result before it is written: y = act(dot + bias[row]) scale + resid, the last two where given
enum { AXQ_ACT_NONE = 0,
       AXQ_ACT_SILU,
       AXQ_ACT_SIGMOID,
       AXQ_ACT_TANH,
       AXQ_ACT_DECAY,     // exp(-exp(v)): the decay factor of a gated recurrence
       AXQ_ACT_SOFTCAP,   // cap * tanh(v / cap)
       AXQ_ACT_RELU2,     // the square of relu
       AXQ_ACT_GLU_GELU };// rows come in groups of AXQ_GLU_GROUP "gate" rows and as many "up" rows: the gate rows' results take
                          // gelu (tanh form); a product of bf16 rows with `out16` goes on to gelu(gate) * up, n / 2 columns
#define AXQ_GLU_GROUP 32

// A weighted mean over what earlier layers left, taken where a layer's result is written:
// out[i] = w[n] y[i] + sum over j < n of w[j] past[j * stride + i]
struct axq_avg { const float *w; const float *past; size_t stride; int n; float *out; };

struct axq_part {
    const uint16_t *w; // bf16 [n][ldw]
    int ldw, n, act;
    int out16;         // row form only: y is bf16
    const float *bias; // [n] or NULL
    const float *mu;   // AXQ_IN_TANH_NORM_MIX: how far this part's input leans to the previous token's
    const float *nw;   // AXQ_IN_LAYER_NORM: this part's norm weight (parts of one launch may have several)
    const void *x;     // row form only: [m][ldx] bf16 or f32
    void *y;           // [n], or [m][ldy]
    int ldy;
    const float *resid;     // where y's are, added; NULL: nothing
    const float *scale;     // row form only: factor of row t at scale[t]; NULL: 1
    const int32_t *sel;     // vector form only: row r is row sel[r / sel_rows] * sel_rows + r % sel_rows of w
    int sel_rows;
    axq_avg avg;            // avg.out == NULL: none
    int blk0;               // filled in by the launchers
};
struct axq_parts {
    axq_part p[AXQ_MAX_PARTS];
    int n_parts, n_blocks;
    float cap;
};

// What happens to a vector before the products of a decode step use it
enum { AXQ_IN_PLAIN = 0,
       AXQ_IN_TANH_NORM,     // tanh(alpha x) nw + nb
       AXQ_IN_TANH_NORM_MIX, // n = that, p = the previous token's (zero at position 0): n + (p - n) mu of the part
       AXQ_IN_RMS_GATE,      // x / sqrt(mean(x^2) + eps) * nw * gate
       AXQ_IN_POLY_NORM,     // c0 N(x) + c1 N(x^2) + c2 N(x^3) + c3, N(z) = z / sqrt(mean(z^2) + eps)
       AXQ_IN_LAYER_NORM,    // (x - mean) / sqrt(mean((x - mean)^2) + eps) * nw of the part
       AXQ_IN_SEGMENTS };    // x and the one weight are put together from axq_in.seg
// A stretch of the input of a product with AXQ_IN_SEGMENTS, `count` times in a row: item i is x[i * ldx ..] times scale[i]
// against the weight at w + (sel ? sel[i] : i) * stride.
struct axq_seg {
    const uint16_t *w;
    int ldw, k, count, ldx;
    size_t stride;
    const int32_t *sel;
    const float *x, *scale;
    int glu;           // x is [groups][2][AXQ_GLU_GROUP]: the products of the two halves
    int step0, steps;  // filled in by the launcher: first step, steps of an item
};
#define AXQ_MAX_SEGS 3
#define AXQ_MAX_SEG_ITEMS 64
struct axq_in {
    const float *x = nullptr;
    int k = 0;
    float eps = 0.f;
    const float *alpha = nullptr, *nw = nullptr, *nb = nullptr; // alpha: one float
    const float *prev = nullptr;    // [k] the previous token's normed input
    const int32_t *pos = nullptr;   // position of this token
    const float *gate = nullptr, *coef = nullptr;
    const int32_t *rows = nullptr;  // norms of rows: output row t is input row rows[t] (NULL: t)
    axq_seg seg[AXQ_MAX_SEGS] = {};
    int n_seg = 0;
};

#define AXQ_DENSE_MAX_K 36864 // widest input of a decode product (it is staged in LDS)

// One vector against the parts.
int axq_dense_gemv(axq_ctx *ctx, int mode, const axq_in &in, axq_parts &parts);
// m rows against the parts; k is padded by the caller's rows to ldx = a multiple of 64 with zeros.
// f32 rows: true 32-bit multiply-adds; bf16 rows: the matrix pipe.
int axq_dense_gemm(axq_ctx *ctx, axq_parts &parts, int m, int k, int ldx, bool f32);
// Rows sorted by the weight they go through (a mixture's experts): weight e is part.w + e * stride.  `tiles` is made on the
// device by axq_moe_sort for the same `bm`: tiles[0] of them, tile i covers slots tiles[4 i + 5] .. tiles[4 i + 6] - 1 and goes
// through weight tiles[4 i + 4].  Row `slot` of the operand is src[slot] (NULL: slot); results are rows of y by slot.
struct axq_groups { const int32_t *tiles, *src; size_t stride; int max_tiles, bm; };
int axq_dense_gemm_rows_per_tile(int rows, int groups, bool f32); // bm for `rows` rows over `groups` weights
int axq_dense_gemm_grouped(axq_ctx *ctx, axq_part &part, const axq_groups &g, int k, int ldx, bool f32);

// ---- row operations of a prompt: xt = bf16 or f32 rows of ldx elements (the tail beyond k zeroed) -----------------
struct axq_rows_out { void *x; int ldx; bool f32; };
int axq_rows_embed(axq_ctx *ctx, const uint16_t *emb16, const float *emb32, const float *pos_table, const int32_t *tok, const int32_t *pos,
                   int pos0, int m, int width, float *h);
// n_mix = 0: the normed rows; else one output per mu[i], n + (p - n) mu, consecutive blocks of `m` rows
int axq_rows_tanh_norm(axq_ctx *ctx, const axq_in &in, int m, bool first, int n_mix, const float *const *mu, axq_rows_out out);
int axq_rows_rms_gate(axq_ctx *ctx, const axq_in &in, int m, int group, axq_rows_out out); // root mean square over groups of `group`
int axq_rows_poly_norm(axq_ctx *ctx, const axq_in &in, int m, axq_rows_out out);
// layer norms of the same rows with one or two weights (nw2 NULL: one), to one or two operands
int axq_rows_layer_norm(axq_ctx *ctx, const axq_in &in, int m, const float *nw1, axq_rows_out out1, const float *nw2, axq_rows_out out2);
// z [m][2 k'] in groups of AXQ_GLU_GROUP gates (activated) and ups -> their products
int axq_rows_glu(axq_ctx *ctx, const float *z, int ldz, int k, int m, axq_rows_out out);
int axq_rows_zero_tail(axq_ctx *ctx, int m, int k, axq_rows_out out);
// prev = the normed input of row m - 1 (what the next token mixes with)
int axq_store_prev(axq_ctx *ctx, const axq_in &in, int m, float *prev);

// ---- linear-state recurrences (axq_linstate.hip) ------------------------------------------------------------------
// S <- diag(w) S + k v^T per head, S f32 [heads][dk][dv].
// w: one constant per head (decay[heads]) or one factor per token, head and key channel (wt [m][heads * dk]).
// o: S^T q after the update, or, with a bonus u [heads][dk], (S + diag(u) k v^T)^T q before it.
struct axq_linstate {
    int heads, dk, dv;
    const float *q, *k, *v, *wt; // rows ld apart
    int ldq, ldk, ldv, ldw;
    const float *decay, *u;
    float *state, *o; // o [m][heads * dv]
    float *seg_state, *seg_decay; // scratch of a prompt cut into segments: AXQ_LINSTATE_SEGS x [heads][dk][dv], x [heads][dk]
};
#define AXQ_LINSTATE_SEGS 16
int axq_linstate_rows(axq_ctx *ctx, const axq_linstate &a, int m, bool first);
// one token; with `norm_w` each head's o is divided by its root mean square and multiplied by norm_w and gate
struct axq_linstate_step {
    axq_linstate a;
    const int32_t *pos;
    const float *t1;       // tanh output of the decay's first product [rank], with
    const uint16_t *w2; int ldw2, rank; const float *w0; // its second weight [heads * dk][ldw2] and offset
    const float *norm_w, *gate; float eps;
    axq_in prev_in; float *prev; // prev != NULL: also store this token's normed input there
};
int axq_linstate_token(axq_ctx *ctx, const axq_linstate_step &s);

// ---- causal attention with sigmoid weights and a distance bias (axq_attn_sigmoid.hip) ------------------------------
struct axq_sig_attn {
    int heads, kv_heads, dim, vdim;
    int cap;                 // positions the cache holds
    float scale, eps;
    const float *qn, *kn;    // [dim] per-head norm weights
    const float *temp;       // [positions] query factor by position
    const float *bias;       // [heads][nt]: what is added to the score of a key n tokens back, n clamped to nt - 1
    int nt;
    void *kc, *vc;           // f16: K [kv][capp][DP], V^T [kv][DVP][capp]; f32: K [kv][cap][dim], V [kv][cap][vdim]
    bool f32;
};
size_t axq_sig_attn_k_bytes(const axq_sig_attn &a);
size_t axq_sig_attn_v_bytes(const axq_sig_attn &a);
size_t axq_sig_attn_q_bytes(const axq_sig_attn &a, int m);   // scratch for the prepared queries of m rows
size_t axq_sig_attn_part_bytes(const axq_sig_attn &a);       // scratch of a decode step
// rows q [m][ldq], k, v (same row stride) at positions pos0.. -> cache, then attention of every row.
int axq_sig_attn_rows(axq_ctx *ctx, const axq_sig_attn &a, const float *q, const float *k, const float *v, int ldq, int ldk, int ldv, int m,
                      int pos0, void *qscratch, axq_rows_out out);
// one token at position *pos -> att f32 [heads * vdim]
int axq_sig_attn_token(axq_ctx *ctx, const axq_sig_attn &a, const float *q, const float *k, const float *v, const int32_t *pos, void *qscratch,
                       float *part, float *att);

// ---- causal softmax attention over a window of tokens and the means of the blocks before it (axq_attn_softmax.hip) ---
struct axq_soft_attn {
    int heads, kv_heads, dim, vdim;
    int cap;                 // positions the cache holds
    int window;              // tokens seen, the newest one included
    int pool;                // tokens of a block that is seen, as its mean key and value, once the window has left it behind; 0: no blocks
    float scale;
    int rot_dims;            // neighbours (2i, 2i + 1) of the first rot_dims dimensions are rotated; 0: none
    const float *rc, *rs;    // [positions][rot_dims / 2] cosines and sines
    void *kc, *vc;           // f16: K [kv][capp][DP], V^T [kv][DVP][capp]; f32: K [kv][cap][dim], V [kv][cap][vdim]
    void *pkc, *pvc;         // the same for the blocks' means, cap / P of them
    bool f32;
};
size_t axq_soft_attn_k_bytes(const axq_soft_attn &a);
size_t axq_soft_attn_v_bytes(const axq_soft_attn &a);
size_t axq_soft_attn_pk_bytes(const axq_soft_attn &a);
size_t axq_soft_attn_pv_bytes(const axq_soft_attn &a);
size_t axq_soft_attn_q_bytes(const axq_soft_attn &a, int m);
size_t axq_soft_attn_part_bytes(const axq_soft_attn &a);
// q [m][ldq], k [m][ldk], v [m][ldv] (v may be k: it is not rotated) at positions pos0.. -> cache, then attention of every row;
// gate [m][heads] (NULL: none) multiplies each head's result
int axq_soft_attn_rows(axq_ctx *ctx, const axq_soft_attn &a, const float *q, const float *k, const float *v, int ldq, int ldk, int ldv,
                       const float *gate, int m, int pos0, void *qscratch, axq_rows_out out);
int axq_soft_attn_token(axq_ctx *ctx, const axq_soft_attn &a, const float *q, const float *k, const float *v, const float *gate,
                        const int32_t *pos, void *qscratch, float *part, float *att);

// ---- mixtures of experts (axq_moe.hip) ----------------------------------------------------------------------------
struct axq_moe_router { int experts, top, groups, keep; };
#define AXQ_MOE_MAX_EXPERTS 1024
// Scores sigmoid(z); of the `groups` equal groups of neighbours the `keep` with the largest sums of their two best scores can
// be chosen from; the `top` best scores there, divided by their sum, are the weights.  sel, wt [m][top].
int axq_moe_route(axq_ctx *ctx, const axq_moe_router &r, const float *z, int ldz, int m, int32_t *sel, float *wt);
// sel [n] -> slots sorted by expert: slot_of [n], src[slot] = entry / top, and the tiles of axq_groups (4 max_tiles + 4 ints)
int axq_moe_max_tiles(int n, int experts, int bm);
int axq_moe_sort(axq_ctx *ctx, const int32_t *sel, int n, int top, int experts, int bm, int32_t *slot_of, int32_t *src, int32_t *tiles);
// y[t] += sum over j of wt[t][j] ye[slot_of[t][j]], then the mean over earlier layers where avg.out is set
int axq_moe_combine(axq_ctx *ctx, const float *ye, const int32_t *slot_of, const float *wt, int top, int m, int width, float *y, const axq_avg &avg);

#ifdef __HIPCC__
__device__ inline float axq_bf16_lo(uint32_t u) { return __builtin_bit_cast(float, u << 16); }
__device__ inline float axq_bf16_hi(uint32_t u) { return __builtin_bit_cast(float, u & 0xFFFF0000u); }
__device__ inline uint16_t axq_to_bf16(float f) {
    const uint32_t u = __builtin_bit_cast(uint32_t, f);
    if ((u & 0x7FFFFFFFu) > 0x7F800000u) return (uint16_t)((u >> 16) | 0x40u);
    return (uint16_t)((u + 0x7FFFu + ((u >> 16) & 1u)) >> 16);
}
__device__ inline float axq_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ inline float axq_act(int act, float v, float cap) {
    switch (act) {
    case AXQ_ACT_SILU: return v * axq_sigmoid(v);
    case AXQ_ACT_SIGMOID: return axq_sigmoid(v);
    case AXQ_ACT_TANH: return tanhf(v);
    case AXQ_ACT_DECAY: return expf(-expf(v));
    case AXQ_ACT_SOFTCAP: return cap * tanhf(v / cap);
    case AXQ_ACT_RELU2: return v > 0.f ? v * v : 0.f;
    default: return v;
    }
}
__device__ inline float axq_gelu_tanh(float v) { return 0.5f * v * (1.0f + tanhf(0.7978845608028654f * fmaf(0.044715f * v * v, v, v))); }
__device__ inline float axq_average(const axq_avg &a, size_t i, float y) {
    float s = 0.f;
    for (int j = 0; j < a.n; j++) s = fmaf(a.w[j], a.past[j * a.stride + i], s);
    return fmaf(a.w[a.n], y, s);
}
// Sum over the 64 lanes; every lane gets it.
__device__ inline float axq_wave_sum(float s) {
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0xB1, 0xf, 0xf, true));  // quad: lanes ^ 1
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0x4E, 0xf, 0xf, true));  // quad: lanes ^ 2
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0x141, 0xf, 0xf, true)); // half-row mirror
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0x140, 0xf, 0xf, true)); // row mirror
    s += __shfl_xor(s, 16);
    s += __shfl_xor(s, 32);
    return s;
}
// Sum over a workgroup of whole waves (at most 16); scratch: 16 floats.
__device__ inline float axq_block_sum(float v, float *scratch) {
    v = axq_wave_sum(v);
    const int wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[wave] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < nw; i++) t += scratch[i];
    return t;
}
#endif
