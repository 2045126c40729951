// Linear-state recurrences: S <- diag(w) S + k v^T per head in f32, read out with q (linear attention with a constant
// decay per head) or, before the update and with a bonus for the current token, with r (time mixing with a decay per
// token, head and key channel).
//
// The columns of S do not depend on each other, so a workgroup takes 16 columns of one head; a column lies across 16
// lanes, every lane keeping dk / 16 of its elements in registers for the whole prompt.  Tokens come through LDS in
// blocks; the next block is requested while the current one is worked on.
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

template <int E, bool TOKEN_DECAY>
__global__ void __launch_bounds__(256) linstate_rows_kernel(axq_linstate a, int m, int first) {
    constexpr int DKP = 16 * E, NV = TOKEN_DECAY ? 3 : 2, TB = E <= 8 ? 16 : (E <= 12 ? 8 : 4);
    constexpr int LOADS = (NV * TB * DKP + 255) / 256; // per thread and block
    __shared__ __attribute__((aligned(16))) float vec[2][NV][TB][DKP];
    __shared__ float val[2][TB][16], os[TB][16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane & 15, cw = lane >> 4;
    const int head = blockIdx.x, c0 = blockIdx.y * 16, mycol = wave * 4 + cw, col = c0 + mycol;
    const bool live = col < a.dv;
    const float *q = a.q + (size_t)head * a.dk, *k = a.k + (size_t)head * a.dk, *v = a.v + (size_t)head * a.dv;
    const float *wt = TOKEN_DECAY ? a.wt + (size_t)head * a.dk : nullptr;
    float *st = a.state + (size_t)head * a.dk * a.dv;

    float S[E], u[E];
#pragma unroll
    for (int i = 0; i < E; i++) {
        const int e = elem_of<E>(g, i);
        S[i] = (!first && live && e < a.dk) ? st[(size_t)e * a.dv + col] : 0.f;
        u[i] = (TOKEN_DECAY && e < a.dk) ? a.u[(size_t)head * a.dk + e] : 0.f;
    }
    const float decay = TOKEN_DECAY ? 0.f : a.decay[head];

    float pre[LOADS], prev_v;
    auto request = [&](int t0) {
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const int idx = tid + i * 256, e = idx % DKP, r = idx / DKP, t = t0 + r % TB, which = r / TB;
            float x = 0.f;
            if (which < NV && t < m && e < a.dk) {
                if (which == 0) x = q[(size_t)t * a.ldq + e];
                else if (which == 1) x = k[(size_t)t * a.ldk + e];
                else x = wt[(size_t)t * a.ldw + e];
            }
            pre[i] = x;
        }
        const int t = t0 + (tid >> 4), c = c0 + (tid & 15);
        prev_v = (tid < TB * 16 && t < m && c < a.dv) ? v[(size_t)t * a.ldv + c] : 0.f;
    };
    auto deposit = [&](int stage) {
        float *dst = &vec[stage][0][0][0];
#pragma unroll
        for (int i = 0; i < LOADS; i++)
            if (tid + i * 256 < NV * TB * DKP) dst[tid + i * 256] = pre[i];
        if (tid < TB * 16) val[stage][tid >> 4][tid & 15] = prev_v;
    };
    request(0);
    deposit(0);
    __syncthreads();
    for (int t0 = 0, stage = 0; t0 < m; t0 += TB, stage ^= 1) {
        if (t0 + TB < m) request(t0 + TB);
        const int nt = m - t0 < TB ? m - t0 : TB;
        for (int t = 0; t < nt; t++) {
            float qe[E], ke[E];
            load_elems<E>(vec[stage][0][t], g, qe);
            load_elems<E>(vec[stage][1][t], g, ke);
            const float vv = val[stage][t][mycol];
            float o = 0.f;
            if (TOKEN_DECAY) {
                float we[E];
                load_elems<E>(vec[stage][NV - 1][t], g, we);
#pragma unroll
                for (int i = 0; i < E; i++) {
                    const float kv = ke[i] * vv;
                    o = fmaf(qe[i], fmaf(u[i], kv, S[i]), o);
                    S[i] = fmaf(we[i], S[i], kv);
                }
            } else {
#pragma unroll
                for (int i = 0; i < E; i++) {
                    S[i] = fmaf(decay, S[i], ke[i] * vv);
                    o = fmaf(qe[i], S[i], o);
                }
            }
            o = row_sum16(o);
            if (g == 0) os[t][mycol] = o;
        }
        if (t0 + TB < m) deposit(stage ^ 1);
        __syncthreads(); // the outputs are complete, the next block is in place
        if (tid < nt * 16 && c0 + (tid & 15) < a.dv)
            a.o[(size_t)(t0 + (tid >> 4)) * a.heads * a.dv + (size_t)head * a.dv + c0 + (tid & 15)] = os[tid >> 4][tid & 15];
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < E; i++) {
        const int e = elem_of<E>(g, i);
        if (live && e < a.dk) st[(size_t)e * a.dv + col] = S[i];
    }
}

template <int E>
int launch_rows(axq_ctx *ctx, const axq_linstate &a, int m, bool first) {
    const dim3 grid(a.heads, (a.dv + 15) / 16);
    if (a.wt) linstate_rows_kernel<E, true><<<grid, 256, 0, ctx->stream>>>(a, m, first ? 1 : 0);
    else linstate_rows_kernel<E, false><<<grid, 256, 0, ctx->stream>>>(a, m, first ? 1 : 0);
    AXQ_LAUNCH_CHECK(ctx, "linstate_rows_kernel");
    return AXQ_OK;
}

// One token.  grid (heads, column blocks of CB): thread = (column, group of key elements); with a head norm one
// workgroup holds the whole head (CB >= dv).  Rows of S are contiguous in the columns.
struct StepArgs {
    axq_linstate_step s;
    int cb;
};

__global__ void __launch_bounds__(512) linstate_token_kernel(StepArgs sa) {
    const axq_linstate_step &s = sa.s;
    const axq_linstate &a = s.a;
    extern __shared__ float sm[];
    __shared__ float scratch[16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nwave = blockDim.x >> 6, head = blockIdx.x;
    const int c0 = blockIdx.y * sa.cb, nc = a.dv - c0 < sa.cb ? a.dv - c0 : sa.cb;
    float *qs = sm, *ks = qs + a.dk, *ws = ks + a.dk, *us = ws + a.dk, *part = us + a.dk; // part [groups][cb]
    const bool first = s.pos[0] == 0;
    for (int e = tid; e < a.dk; e += blockDim.x) {
        qs[e] = a.q[(size_t)head * a.dk + e];
        ks[e] = a.k[(size_t)head * a.dk + e];
        us[e] = a.u ? a.u[(size_t)head * a.dk + e] : 0.f;
        if (!s.t1) ws[e] = a.decay[head];
    }
    if (s.t1) { // w = exp(-exp(W2 t1 + w0)), a wave per key channel
        for (int e = wave; e < a.dk; e += nwave) {
            const uint16_t *row = s.w2 + (size_t)(head * a.dk + e) * s.ldw2;
            float z = 0.f;
            for (int r = lane; r < s.rank; r += 64) z = fmaf(axq_bf16_lo(row[r]), s.t1[r], z);
            z = axq_wave_sum(z);
            if (lane == 0) ws[e] = expf(-expf(z + s.w0[(size_t)head * a.dk + e]));
        }
    }
    __syncthreads();
    const int col = tid % sa.cb, grp = tid / sa.cb, ngrp = blockDim.x / sa.cb;
    float o = 0.f;
    if (grp < ngrp && col < nc) {
        const float vv = a.v[(size_t)head * a.dv + c0 + col];
        float *st = a.state + (size_t)head * a.dk * a.dv + c0 + col;
        for (int e0 = grp; e0 < a.dk; e0 += 4 * ngrp) {
            float old[4];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int e = e0 + i * ngrp;
                old[i] = (!first && e < a.dk) ? st[(size_t)e * a.dv] : 0.f;
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int e = e0 + i * ngrp;
                if (e < a.dk) {
                    const float kv = ks[e] * vv, nw = fmaf(ws[e], old[i], kv);
                    o = fmaf(qs[e], a.u ? fmaf(us[e], kv, old[i]) : nw, o);
                    st[(size_t)e * a.dv] = nw;
                }
            }
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
