// Linear-state recurrences: S <- diag(w) S + k v^T per head in f32, read out with q (linear attention with a constant
// decay per head) or, before the update and with a bonus for the current token, with r (time mixing with a decay per
// token, head and key channel).
//
// The columns of S do not depend on each other, so a workgroup takes 16 columns of one head; a column lies across 16
// lanes, every lane keeping dk / 16 of its elements in registers for the whole prompt.  Tokens come through LDS in
// blocks; the next block is requested while the current one is worked on.  Where heads x columns do not fill the chip, the
// prompt is cut into segments: their states from zero, a scan over them (the update is linear in the state), then all
// segments side by side from the states they start in.
#include "axq_dense.h"

namespace {

// Sum over aligned groups of 16 lanes; every lane gets it.
__device__ inline float row_sum16(float s) {
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0xB1, 0xf, 0xf, true));
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0x4E, 0xf, 0xf, true));
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0x141, 0xf, 0xf, true));
    s += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, s), 0x140, 0xf, 0xf, true));
    return s;
}

// E elements of a key column per lane.  Lane g of a column owns elements 64 i + 4 g .. + 3 when E is a multiple of 4
// (16-byte LDS reads), else 16 i + g.
template <int E>
__device__ inline int elem_of(int g, int i) { return E % 4 == 0 ? 64 * (i >> 2) + 4 * g + (i & 3) : 16 * i + g; }

template <int E>
__device__ inline void load_elems(const float *row, int g, float (&out)[E]) {
    if (E % 4 == 0) {
#pragma unroll
        for (int i = 0; i < E / 4; i++) {
            const float4 v = *reinterpret_cast<const float4 *>(row + 64 * i + 4 * g);
            out[4 * i] = v.x; out[4 * i + 1] = v.y; out[4 * i + 2] = v.z; out[4 * i + 3] = v.w;
        }
    } else {
#pragma unroll
        for (int i = 0; i < E; i++) out[i] = row[16 * i + g];
    }
}

// Tokens of a group are independent but for the state: their vectors are read ahead, their outputs reduced together.
template <int E, bool TOKEN_DECAY, bool STATE_ONLY, bool VEC>
__global__ void __launch_bounds__(256) linstate_rows_kernel(axq_linstate a, int m_all, int first, int seg_len) {
    constexpr int DKP = 16 * E, NV = TOKEN_DECAY ? 3 : 2, G = E <= (TOKEN_DECAY ? 5 : 8) ? 4 : 2, TB = E <= 8 ? 16 : (E <= 12 ? 8 : 4);
    constexpr int W = VEC ? 4 : 1, LOADS = (NV * TB * DKP / W + 255) / 256; // per thread and block
    __shared__ __attribute__((aligned(16))) float vec[2][NV][TB][DKP];
    __shared__ __attribute__((aligned(16))) float val[2][16][TB], os[16][TB + 1]; // by column
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane & 15, cw = lane >> 4;
    const int head = blockIdx.x, c0 = blockIdx.y * 16, mycol = wave * 4 + cw, col = c0 + mycol;
    const bool live = col < a.dv;
    const int seg = blockIdx.z, t_beg = seg * seg_len, m = m_all - t_beg < seg_len ? m_all - t_beg : seg_len;
    const float *q = a.q + (size_t)t_beg * a.ldq + (size_t)head * a.dk, *k = a.k + (size_t)t_beg * a.ldk + (size_t)head * a.dk;
    const float *v = a.v + (size_t)t_beg * a.ldv + (size_t)head * a.dv;
    const float *wt = TOKEN_DECAY ? a.wt + (size_t)t_beg * a.ldw + (size_t)head * a.dk : nullptr;
    const size_t head_state = (size_t)head * a.dk * a.dv, all_states = (size_t)a.heads * a.dk * a.dv;
    float *o_out = a.o + (size_t)t_beg * a.heads * a.dv;
    const bool cut = STATE_ONLY || seg_len < m_all;
    float *st = (cut ? a.seg_state + seg * all_states : a.state) + head_state;
    first = STATE_ONLY || (first && !cut); // of several segments each starts in a state of its own

    float S[E], u[E], wp[STATE_ONLY ? E : 1];
#pragma unroll
    for (int i = 0; i < (STATE_ONLY ? E : 1); i++) wp[i] = 1.f;
#pragma unroll
    for (int i = 0; i < E; i++) {
        const int e = elem_of<E>(g, i);
        S[i] = (!first && live && e < a.dk) ? st[(size_t)e * a.dv + col] : 0.f;
        u[i] = (TOKEN_DECAY && e < a.dk) ? a.u[(size_t)head * a.dk + e] : 0.f;
    }
    const float decay = TOKEN_DECAY ? 0.f : a.decay[head];

    // tokens beyond the last: k = 0 and a decay of 1 leave the state as it is
    float pre[LOADS][W], pre_v;
    auto request = [&](int t0) {
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const int idx = (tid + i * 256) * W, e = idx % DKP, r = idx / DKP, t = t0 + r % TB, which = r / TB;
            const bool there = which < NV && t < m && e < a.dk;
            const float *src = which == 0 ? q + (size_t)t * a.ldq + e : k + (size_t)t * a.ldk + e;
            if constexpr (TOKEN_DECAY) src = which == 2 ? wt + (size_t)t * a.ldw + e : src;
            const float none = TOKEN_DECAY && which == 2 ? 1.f : 0.f;
            if (VEC) {
                const float4 x = there ? *reinterpret_cast<const float4 *>(src) : make_float4(none, none, none, none);
                pre[i][0] = x.x; pre[i][1 % W] = x.y; pre[i][2 % W] = x.z; pre[i][3 % W] = x.w;
            } else {
                pre[i][0] = there ? *src : none;
            }
        }
        const int t = t0 + (tid >> 4), c = c0 + (tid & 15);
        pre_v = (tid < TB * 16 && t < m && c < a.dv) ? v[(size_t)t * a.ldv + c] : 0.f;
    };
    auto deposit = [&](int stage) {
        float *dst = &vec[stage][0][0][0];
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const int idx = (tid + i * 256) * W;
            if (idx < NV * TB * DKP) {
                if (VEC) *reinterpret_cast<float4 *>(dst + idx) = make_float4(pre[i][0], pre[i][1 % W], pre[i][2 % W], pre[i][3 % W]);
                else dst[idx] = pre[i][0];
            }
        }
        if (tid < TB * 16) val[stage][tid & 15][tid >> 4] = pre_v;
    };
    struct Group { float q[G][STATE_ONLY ? 1 : E], k[G][E], w[G][TOKEN_DECAY ? E : 1], v[G]; };
    auto read = [&](int stage, int t, Group &x) {
#pragma unroll
        for (int i = 0; i < G; i++) {
            if constexpr (!STATE_ONLY) load_elems<E>(vec[stage][0][t + i], g, x.q[i]);
            load_elems<E>(vec[stage][1][t + i], g, x.k[i]);
            if constexpr (TOKEN_DECAY) load_elems<E>(vec[stage][NV - 1][t + i], g, x.w[i]);
            x.v[i] = val[stage][mycol][t + i];
        }
    };
    auto work = [&](int t, int nt, const Group &x) {
        float o[G];
#pragma unroll
        for (int j = 0; j < G; j++) {
            float s = 0.f;
            const bool token = TOKEN_DECAY || t + j < nt; // a constant decay must not touch the state beyond the last token
#pragma unroll
            for (int i = 0; i < E; i++) {
                const float kv = x.k[j][i] * x.v[j];
                if constexpr (STATE_ONLY) {
                    float w = decay; // segments of a state-only pass are whole blocks
                    if constexpr (TOKEN_DECAY) w = x.w[j][i];
                    S[i] = fmaf(w, S[i], kv);
                    wp[i] *= w;
                } else if constexpr (TOKEN_DECAY) {
                    s = fmaf(x.q[j][i], fmaf(u[i], kv, S[i]), s);
                    S[i] = fmaf(x.w[j][i], S[i], kv);
                } else {
                    S[i] = fmaf(token ? decay : 1.f, S[i], kv);
                    s = fmaf(x.q[j][i], S[i], s);
                }
            }
            o[j] = s;
        }
        if constexpr (!STATE_ONLY) {
#pragma unroll
            for (int j = 0; j < G; j++) o[j] = row_sum16(o[j]);
            if (g == 0) {
#pragma unroll
                for (int j = 0; j < G; j++) os[mycol][t + j] = o[j];
            }
        }
    };
    request(0);
    deposit(0);
    __syncthreads();
    for (int t0 = 0, stage = 0; t0 < m; t0 += TB, stage ^= 1) {
        if (t0 + TB < m) request(t0 + TB);
        const int nt = m - t0 < TB ? m - t0 : TB;
        Group ga, gb;
        read(stage, 0, ga);
#pragma unroll
        for (int t = 0; t < TB; t += 2 * G) {
            read(stage, t + G, gb);
            work(t, nt, ga);
            if (t + 2 * G < TB) read(stage, t + 2 * G, ga);
            work(t + G, nt, gb);
        }
        if (t0 + TB < m) deposit(stage ^ 1);
        __syncthreads(); // the outputs are complete, the next block is in place
        if (!STATE_ONLY && tid < nt * 16 && c0 + (tid & 15) < a.dv)
            o_out[(size_t)(t0 + (tid >> 4)) * a.heads * a.dv + (size_t)head * a.dv + c0 + (tid & 15)] = os[tid & 15][tid >> 4];
        __syncthreads();
    }
    if (!STATE_ONLY && cut) {
        if (t_beg + m < m_all) return;
        st = a.state + head_state; // the last segment leaves the state behind
    }
#pragma unroll
    for (int i = 0; i < E; i++) {
        const int e = elem_of<E>(g, i);
        if (live && e < a.dk) st[(size_t)e * a.dv + col] = S[i];
        if constexpr (STATE_ONLY)
            if (col == 0 && e < a.dk) a.seg_decay[((size_t)seg * a.heads + head) * a.dk + e] = wp[i];
    }
}

// seg_state[s] <- the state segment s starts in, given the segments' own contributions
__global__ void __launch_bounds__(256) linstate_scan_kernel(axq_linstate a, int segs, int first) {
    const size_t n = (size_t)a.heads * a.dk * a.dv, i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const size_t hk = i / a.dv;
    float run = first ? 0.f : a.state[i];
    for (int s = 0; s < segs; s++) {
        const float own = s + 1 < segs ? a.seg_state[s * n + i] : 0.f, w = s + 1 < segs ? a.seg_decay[(size_t)s * a.heads * a.dk + hk] : 0.f;
        a.seg_state[s * n + i] = run;
        run = fmaf(w, run, own);
    }
}

template <int E, bool TOKEN_DECAY, bool VEC>
int launch_rows_t(axq_ctx *ctx, const axq_linstate &a, int m, bool first, int segs) {
    const int cols = (a.dv + 15) / 16, len = segs > 1 ? ((m + segs - 1) / segs + 15) / 16 * 16 : m;
    segs = (m + len - 1) / len;
    if (segs > 1) {
        linstate_rows_kernel<E, TOKEN_DECAY, true, VEC><<<dim3(a.heads, cols, segs - 1), 256, 0, ctx->stream>>>(a, m, 1, len);
        linstate_scan_kernel<<<(unsigned)(((size_t)a.heads * a.dk * a.dv + 255) / 256), 256, 0, ctx->stream>>>(a, segs, first ? 1 : 0);
    }
    linstate_rows_kernel<E, TOKEN_DECAY, false, VEC><<<dim3(a.heads, cols, segs), 256, 0, ctx->stream>>>(a, m, first ? 1 : 0, len);
    AXQ_LAUNCH_CHECK(ctx, "linstate_rows_kernel");
    return AXQ_OK;
}

template <int E>
int launch_rows(axq_ctx *ctx, const axq_linstate &a, int m, bool first) {
    const int wgs = a.heads * ((a.dv + 15) / 16);
    int segs = 1;
    if (a.seg_state && wgs < ctx->prop.multiProcessorCount) {
        segs = 2 * ctx->prop.multiProcessorCount / wgs;
        if (segs > m / 64) segs = m / 64;
        if (segs > AXQ_LINSTATE_SEGS) segs = AXQ_LINSTATE_SEGS;
        if (segs < 1) segs = 1;
    }
    auto aligned = [](const void *p, int ld) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0 && ld % 4 == 0; };
    const bool vec = a.dk % 4 == 0 && aligned(a.q, a.ldq) && aligned(a.k, a.ldk) && (!a.wt || aligned(a.wt, a.ldw));
    if (a.wt) return vec ? launch_rows_t<E, true, true>(ctx, a, m, first, segs) : launch_rows_t<E, true, false>(ctx, a, m, first, segs);
    return vec ? launch_rows_t<E, false, true>(ctx, a, m, first, segs) : launch_rows_t<E, false, false>(ctx, a, m, first, segs);
}

// One token.  grid (heads, column blocks of CB): thread = (column, group of key elements); with a head norm one
// workgroup holds the whole head (CB >= dv).  Rows of S are contiguous in the columns.
struct StepArgs {
    axq_linstate_step s;
    int cb;
};

constexpr int TOKEN_PRE = 16; // state elements a thread requests before anything else

__global__ void __launch_bounds__(512) linstate_token_kernel(StepArgs sa) {
    const axq_linstate_step &s = sa.s;
    const axq_linstate &a = s.a;
    extern __shared__ float sm[];
    __shared__ float scratch[16];
    const int tid = threadIdx.x, head = blockIdx.x;
    const int c0 = blockIdx.y * sa.cb, nc = a.dv - c0 < sa.cb ? a.dv - c0 : sa.cb;
    float *qs = sm, *ks = qs + a.dk, *ws = ks + a.dk, *us = ws + a.dk, *part = us + a.dk; // part [groups][cb]
    const bool first = s.pos[0] == 0;
    const int col = tid % sa.cb, grp = tid / sa.cb, ngrp = blockDim.x / sa.cb;
    const bool live = grp < ngrp && col < nc;
    float *st = a.state + (size_t)head * a.dk * a.dv + c0 + (live ? col : 0);
    float old[TOKEN_PRE];
#pragma unroll
    for (int i = 0; i < TOKEN_PRE; i++) {
        const int e = grp + i * ngrp;
        old[i] = (!first && live && e < a.dk) ? st[(size_t)e * a.dv] : 0.f;
    }
    const float vv = live ? a.v[(size_t)head * a.dv + c0 + col] : 0.f;
    for (int e = tid; e < a.dk; e += blockDim.x) {
        qs[e] = a.q[(size_t)head * a.dk + e];
        ks[e] = a.k[(size_t)head * a.dk + e];
        us[e] = a.u ? a.u[(size_t)head * a.dk + e] : 0.f;
        if (!s.t1) ws[e] = a.decay[head];
    }
    if (s.t1) { // w = exp(-exp(W2 t1 + w0)), eight lanes per key channel, 16 bytes of its row at a time
        const int sub = tid & 7;
        for (int e0 = 0; e0 < a.dk; e0 += blockDim.x >> 3) {
            const int e = e0 + (tid >> 3);
            float z = 0.f;
            if (e < a.dk) {
                const uint16_t *row = s.w2 + (size_t)(head * a.dk + e) * s.ldw2;
                for (int r = sub * 8; r < s.rank; r += 64) {
                    const uint4 w = *reinterpret_cast<const uint4 *>(row + r);
                    const uint32_t ww[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
                    for (int i = 0; i < 8; i++)
                        if (r + i < s.rank) z = fmaf(i & 1 ? axq_bf16_hi(ww[i >> 1]) : axq_bf16_lo(ww[i >> 1]), s.t1[r + i], z);
                }
            }
            z += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, z), 0xB1, 0xf, 0xf, true));
            z += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, z), 0x4E, 0xf, 0xf, true));
            z += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, z), 0x141, 0xf, 0xf, true));
            if (e < a.dk && sub == 0) ws[e] = expf(-expf(z + s.w0[(size_t)head * a.dk + e]));
        }
    }
    __syncthreads();
    float o = 0.f;
    auto update = [&](int e, float before) {
        const float kv = ks[e] * vv, now = fmaf(ws[e], before, kv);
        o = fmaf(qs[e], a.u ? fmaf(us[e], kv, before) : now, o);
        st[(size_t)e * a.dv] = now;
    };
    if (live) {
#pragma unroll
        for (int i = 0; i < TOKEN_PRE; i++)
            if (grp + i * ngrp < a.dk) update(grp + i * ngrp, old[i]);
        for (int e0 = grp + TOKEN_PRE * ngrp; e0 < a.dk; e0 += 8 * ngrp) {
            float more[8];
#pragma unroll
            for (int i = 0; i < 8; i++) more[i] = (!first && e0 + i * ngrp < a.dk) ? st[(size_t)(e0 + i * ngrp) * a.dv] : 0.f;
#pragma unroll
            for (int i = 0; i < 8; i++)
                if (e0 + i * ngrp < a.dk) update(e0 + i * ngrp, more[i]);
        }
    }
    if (grp < ngrp) part[grp * sa.cb + col] = o;
    __syncthreads();
    float t = 0.f;
    if (tid < nc)
        for (int i = 0; i < ngrp; i++) t += part[i * sa.cb + tid];
    if (s.norm_w) {
        const float ss = axq_block_sum(tid < nc ? t * t : 0.f, scratch);
        const float inv = 1.0f / sqrtf(ss / (float)a.dv + s.eps);
        if (tid < nc) t = t * inv * s.norm_w[(size_t)head * a.dv + tid] * s.gate[(size_t)head * a.dv + tid];
    }
    if (tid < nc) a.o[(size_t)head * a.dv + c0 + tid] = t;
    if (s.prev && blockIdx.y == 0) { // the products of this step have read the previous token's input
        const int per = (s.prev_in.k + a.heads - 1) / a.heads, e1 = (head + 1) * per < s.prev_in.k ? (head + 1) * per : s.prev_in.k;
        for (int e = head * per + tid; e < e1; e += blockDim.x)
            s.prev[e] = tanhf(s.prev_in.alpha[0] * s.prev_in.x[e]) * s.prev_in.nw[e] + s.prev_in.nb[e];
    }
}

} // namespace

int axq_linstate_rows(axq_ctx *ctx, const axq_linstate &a, int m, bool first) {
    const int e = (a.dk + 15) / 16;
    if (a.dk < 1 || a.dv < 1 || a.heads < 1 || e > 16 || m < 1)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: a linear-state head takes key sizes up to 256, got %d", a.dk);
    switch (e) {
    case 1: return launch_rows<1>(ctx, a, m, first);
    case 2: return launch_rows<2>(ctx, a, m, first);
    case 3: return launch_rows<3>(ctx, a, m, first);
    case 4: return launch_rows<4>(ctx, a, m, first);
    case 5: return launch_rows<5>(ctx, a, m, first);
    case 6: return launch_rows<6>(ctx, a, m, first);
    case 7: case 8: return launch_rows<8>(ctx, a, m, first);
    case 9: case 10: case 11: case 12: return launch_rows<12>(ctx, a, m, first);
    default: return launch_rows<16>(ctx, a, m, first);
    }
}

int axq_linstate_token(axq_ctx *ctx, const axq_linstate_step &s) {
    if (s.a.dk < 1 || s.a.dk > 256 || s.a.dv < 1 || (s.norm_w && s.a.dv > 512))
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: a linear-state head of %d x %d", s.a.dk, s.a.dv);
    StepArgs sa;
    sa.s = s;
    // whole heads where the head's norm needs them, else 32 columns (128 bytes of a state row) per workgroup
    sa.cb = s.norm_w ? (s.a.dv + 15) / 16 * 16 : (s.a.dv < 32 ? s.a.dv : 32);
    const int threads = s.norm_w ? 512 : 256, ngrp = threads / sa.cb;
    const size_t lds = (size_t)(4 * s.a.dk + ngrp * sa.cb) * sizeof(float);
    linstate_token_kernel<<<dim3(s.a.heads, (s.a.dv + sa.cb - 1) / sa.cb), threads, lds, ctx->stream>>>(sa);
    AXQ_LAUNCH_CHECK(ctx, "linstate_token_kernel");
    return AXQ_OK;
}
