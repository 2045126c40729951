// Causal attention whose weights are sigmoids of the scores, not normalised over the keys, with per-head RMS norms on
// queries and keys, a query factor by position and a learned bias by distance:
//   w_ij = sigmoid(scale (q_i . k_j) + bias[h][min(i - j, nt - 1)]),   o_i = sum_j w_ij v_j.
// Without a normaliser partial sums over ranges of keys just add up: no running maximum, no rescaling.
#include "axq_attn_tiles.h"

namespace {

struct Args {
    axq_sig_attn a;
    const float *q, *k, *v;
    int ldq, ldk, ldv;
    int m, pos0;
    const int32_t *pos; // != NULL: one row at *pos
    int capp, dp, dvp;  // f16 cache
    void *qs;           // prepared queries: f16 [m][heads][dp] or f32 [m][heads][dim]
};

// grid (heads + 2 kv_heads, rows), one wave: query head -> normed, scaled by position; key head -> normed, cache; value -> cache
template <bool F32>
__global__ void __launch_bounds__(64) prep_kernel(Args g) {
    const axq_sig_attn &a = g.a;
    const int t = blockIdx.y, lane = threadIdx.x, p = g.pos ? g.pos[0] : g.pos0 + t;
    int h = blockIdx.x;
    if (h < a.heads) {
        const float *q = g.q + (size_t)t * g.ldq + (size_t)h * a.dim;
        float ss = 0.f;
        for (int e = lane; e < a.dim; e += 64) ss = fmaf(q[e], q[e], ss);
        ss = axq_wave_sum(ss);
        const float inv = 1.0f / sqrtf(ss / (float)a.dim + a.eps), temp = a.temp[p];
        if (F32) {
            float *o = reinterpret_cast<float *>(g.qs) + ((size_t)t * a.heads + h) * a.dim;
            for (int e = lane; e < a.dim; e += 64) o[e] = q[e] * inv * a.qn[e] * temp;
        } else {
            _Float16 *o = reinterpret_cast<_Float16 *>(g.qs) + ((size_t)t * a.heads + h) * g.dp;
            for (int e = lane; e < g.dp; e += 64) o[e] = e < a.dim ? to_half(q[e] * inv * a.qn[e] * temp) : (_Float16)0.f;
        }
        return;
    }
    h -= a.heads;
    if (h < a.kv_heads) {
        const float *k = g.k + (size_t)t * g.ldk + (size_t)h * a.dim;
        float ss = 0.f;
        for (int e = lane; e < a.dim; e += 64) ss = fmaf(k[e], k[e], ss);
        ss = axq_wave_sum(ss);
        const float inv = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
        if (F32) {
            float *o = reinterpret_cast<float *>(a.kc) + ((size_t)h * a.cap + p) * a.dim;
            for (int e = lane; e < a.dim; e += 64) o[e] = k[e] * inv * a.kn[e];
        } else {
            _Float16 *o = reinterpret_cast<_Float16 *>(a.kc) + ((size_t)h * g.capp + p) * g.dp;
            for (int e = lane; e < a.dim; e += 64) o[e] = to_half(k[e] * inv * a.kn[e]); // the padding stays zero
        }
        return;
    }
    h -= a.kv_heads;
    const float *v = g.v + (size_t)t * g.ldv + (size_t)h * a.vdim;
    if (F32) {
        float *o = reinterpret_cast<float *>(a.vc) + ((size_t)h * a.cap + p) * a.vdim;
        for (int e = lane; e < a.vdim; e += 64) o[e] = v[e];
    } else {
        _Float16 *o = reinterpret_cast<_Float16 *>(a.vc) + (size_t)h * g.dvp * g.capp + value_slot(p);
        for (int e = lane; e < a.vdim; e += 64) o[(size_t)e * g.capp] = to_half(v[e]);
    }
}

__global__ void __launch_bounds__(256) append_values_kernel(Args g) { append_values(g.v, g.ldv, g.a.vdim, g.m, g.pos0, g.a.vc, g.dvp, g.capp); }

// Rows against the f32 cache: grid (heads, rows).  256 keys at a time: scores by thread, then the value sum by element.
__global__ void __launch_bounds__(256) rows_f32_kernel(Args g, axq_rows_out out) {
    extern __shared__ float sm[];
    const axq_sig_attn &a = g.a;
    const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, p = g.pos ? g.pos[0] : g.pos0 + t;
    const int kvh = h / (a.heads / a.kv_heads), ng = 256 / a.vdim > 0 ? 256 / a.vdim : 1;
    float *qs = sm, *w = qs + a.dim, *red = w + 256; // red [ng][vdim]
    const float *q = reinterpret_cast<const float *>(g.qs) + ((size_t)t * a.heads + h) * a.dim;
    const float *kc = reinterpret_cast<const float *>(a.kc) + (size_t)kvh * a.cap * a.dim;
    const float *vc = reinterpret_cast<const float *>(a.vc) + (size_t)kvh * a.cap * a.vdim;
    const float *bias = a.bias + (size_t)h * a.nt;
    for (int e = tid; e < a.dim; e += 256) qs[e] = q[e];
    for (int e = tid; e < ng * a.vdim; e += 256) red[e] = 0.f;
    __syncthreads();
    for (int j0 = 0; j0 <= p; j0 += 256) {
        const int j = j0 + tid;
        float wt = 0.f;
        if (j <= p) {
            float s = 0.f;
            for (int e = 0; e < a.dim; e++) s = fmaf(qs[e], kc[(size_t)j * a.dim + e], s);
            const int n = p - j < a.nt ? p - j : a.nt - 1;
            wt = axq_sigmoid(fmaf(s, a.scale, bias[n]));
        }
        w[tid] = wt;
        __syncthreads();
        const int n = p + 1 - j0 < 256 ? p + 1 - j0 : 256;
        for (int i = tid; i < ng * a.vdim; i += 256) {
            const int e = i % a.vdim, grp = i / a.vdim;
            float o = red[i];
            for (int jj = grp; jj < n; jj += ng) o = fmaf(w[jj], vc[(size_t)(j0 + jj) * a.vdim + e], o);
            red[i] = o;
        }
        __syncthreads();
    }
    for (int e = tid; e < a.vdim; e += 256) {
        float o = 0.f;
        for (int grp = 0; grp < ng; grp++) o += red[grp * a.vdim + e];
        if (out.f32) reinterpret_cast<float *>(out.x)[(size_t)t * out.ldx + (size_t)h * a.vdim + e] = o;
        else reinterpret_cast<uint16_t *>(out.x)[(size_t)t * out.ldx + (size_t)h * a.vdim + e] = axq_to_bf16(o);
    }
}

// Rows against the f16 cache on the matrix pipe.  A wave takes 32 "virtual queries" (row, query head of the group),
// which are lanes (column lane % 32) all the way through:
//   S^T = K Q^T (32 keys x 32 queries), A = key rows, B = queries;
//   P^T = sigmoid(..) as f16: the accumulator of a lane holds keys 8 i + 4 (lane / 32) + 0..3, and the second product
//         sums over the keys in that very order (value_slot), so P needs no exchange of lanes;
//   O^T += V^T P^T, A = rows of the transposed values.
// The four waves of a workgroup walk the same keys, 64 at a time, through LDS (two stages, filled straight from memory;
// the 16-byte pieces of a row are exchanged by row % 8 so that operand reads use all banks).  Workgroups with the longest
// ranges start first.
template <int KS, int DB>
__global__ void __launch_bounds__(256, KS + DB > 20 ? 1 : 2) rows_mfma_kernel(Args g, axq_rows_out out) {
    constexpr int DP = KS * 16, DVP = DB * 32, KC = DP / 8; // KC: 16-byte pieces of a key row
    constexpr int KH = 64 * DP, STAGE = KH + DVP * 64;       // halfs of a key tile, of a stage
    extern __shared__ __attribute__((aligned(16))) _Float16 tiles[];
    const axq_sig_attn &a = g.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 31, lh = lane >> 5;
    const int kvh = blockIdx.x, rep = a.heads / a.kv_heads, wg = (int)gridDim.y - 1 - (int)blockIdx.y;
    const int total = g.m * rep, vq0 = (wg * 4 + wave) * 32;
    const int vq = vq0 + li, vqc = vq < total ? vq : total - 1;
    const int row = vqc / rep, h = kvh * rep + vqc % rep, p = g.pos0 + row;
    const int last = vq0 + 31 < total ? vq0 + 31 : total - 1, p_min = g.pos0 + (vq0 < total ? vq0 : total - 1) / rep, p_max = g.pos0 + last / rep;
    const int wg_last = wg * 128 + 127 < total ? wg * 128 + 127 : total - 1, wg_max = g.pos0 + wg_last / rep;
    const _Float16 *kc = reinterpret_cast<const _Float16 *>(a.kc) + (size_t)kvh * g.capp * DP;
    const _Float16 *vc = reinterpret_cast<const _Float16 *>(a.vc) + (size_t)kvh * DVP * g.capp;
    const float *bias = a.bias + (size_t)h * a.nt;
    const float far = bias[a.nt - 1], scale = a.scale;
    const _Float16 *gk[DP / 32], *gv[DB];
#pragma unroll
    for (int i = 0; i < DP / 32; i++) {
        const int idx = (i * 4 + wave) * 64 + lane, r = idx / KC, c = (idx % KC) ^ (r & 7);
        gk[i] = kc + (size_t)r * DP + c * 8;
    }
#pragma unroll
    for (int i = 0; i < DB; i++) {
        const int idx = (i * 4 + wave) * 64 + lane, r = idx >> 3, c = (idx & 7) ^ (r & 7);
        gv[i] = vc + (size_t)r * g.capp + c * 8;
    }
    auto fetch = [&](int stage, int j0) { // rows up to capp, a multiple of 64, exist
        _Float16 *lk = tiles + stage * STAGE, *lv = lk + KH;
#pragma unroll
        for (int i = 0; i < DP / 32; i++)
            __builtin_amdgcn_global_load_lds((gbl_void *)(gk[i] + (size_t)j0 * DP), (lds_void *)(lk + (i * 4 + wave) * 512), 16, 0, 0);
#pragma unroll
        for (int i = 0; i < DB; i++)
            __builtin_amdgcn_global_load_lds((gbl_void *)(gv[i] + j0), (lds_void *)(lv + (i * 4 + wave) * 512), 16, 0, 0);
    };
    half8 qf[KS];
    {
        const _Float16 *q = reinterpret_cast<const _Float16 *>(g.qs) + ((size_t)row * a.heads + h) * DP + lh * 8;
#pragma unroll
        for (int ks = 0; ks < KS; ks++) qf[ks] = *reinterpret_cast<const half8 *>(q + ks * 16);
    }
    f32x16 O[DB];
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
        for (int r = 0; r < 16; r++) O[db][r] = 0.f;
    constexpr float LOG2E = 1.4426950408889634f;
    fetch(0, 0);
    for (int t0 = 0, stage = 0; t0 <= wg_max; t0 += 64, stage ^= 1) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); // this tile is in LDS ...
        __syncthreads();                                  // ... of every wave, and nobody reads the other stage any more
        if (t0 + 64 <= wg_max) fetch(stage ^ 1, t0 + 64);
        const _Float16 *lk = tiles + stage * STAGE, *lv = lk + KH;
#pragma unroll
        for (int sub = 0; sub < 2; sub++) {
            const int j0 = t0 + sub * 32;
            if (j0 > p_max) break;
            f32x16 S;
#pragma unroll
            for (int r = 0; r < 16; r++) S[r] = 0.f;
#pragma unroll
            for (int ks = 0; ks < KS; ks++) {
                const half8 kf = *reinterpret_cast<const half8 *>(lk + (sub * 32 + li) * DP + (((ks * 2 + lh) ^ (li & 7)) << 3));
                S = __builtin_amdgcn_mfma_f32_32x32x16_f16(kf, qf[ks], S, 0, 0, 0);
            }
            if (p_min - (j0 + 31) >= a.nt - 1) { // every key of the tile is in the last bucket of every query
#pragma unroll
                for (int r = 0; r < 16; r++) S[r] = fmaf(S[r], scale, far);
            } else {
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    const int n = p - (j0 + acc_row(r, lane));
                    const float b = bias[n < 0 ? 0 : (n < a.nt ? n : a.nt - 1)];
                    S[r] = n >= 0 ? fmaf(S[r], scale, b) : -INFINITY;
                }
            }
            half8 pf[2];
#pragma unroll
            for (int r = 0; r < 16; r++)
                pf[r >> 3][r & 7] = (_Float16)(PSCALE * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * S[r])));
#pragma unroll
            for (int ks = 0; ks < 2; ks++)
#pragma unroll
                for (int db = 0; db < DB; db++) {
                    const half8 vf = *reinterpret_cast<const half8 *>(lv + (db * 32 + li) * 64 + (((sub * 4 + ks * 2 + lh) ^ (li & 7)) << 3));
                    O[db] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, pf[ks], O[db], 0, 0, 0);
                }
        }
    }
    if (vq >= total) return;
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int e = db * 32 + acc_row(r, lane);
            if (e < a.vdim) {
                const float o = O[db][r] * (1.0f / PSCALE);
                const size_t i = (size_t)row * out.ldx + (size_t)h * a.vdim + e;
                if (out.f32) reinterpret_cast<float *>(out.x)[i] = o;
                else reinterpret_cast<uint16_t *>(out.x)[i] = axq_to_bf16(o);
            }
        }
}

// One token, f16 cache: workgroup (kv head, split) takes positions [64 split, 64 split + 64) for all query heads of the
// group.  The one whose range holds the newest position first appends that position's key and value.  Workgroups beyond
// the newest position leave at once (the grid is sized for the whole cache so that the launch can sit in a graph).
template <int DP>
__global__ void __launch_bounds__(256) token_partial_kernel(Args g, float *part) {
    extern __shared__ __attribute__((aligned(16))) float sm2[];
    constexpr int NK = DP / 32; // 16-byte pieces of a key per lane: four lanes take a position's pieces in turn
    const axq_sig_attn &a = g.a;
    const int kvh = blockIdx.x, split = blockIdx.y, p = g.pos[0], p0 = split * CHUNK;
    if (p0 > p) return;
    const int rep = a.heads / a.kv_heads, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    float *qs = sm2, *ws = qs + (size_t)rep * DP; // [rep][DP], [rep][CHUNK] (columns in value_slot order)
    _Float16 *kc = reinterpret_cast<_Float16 *>(a.kc) + (size_t)kvh * g.capp * DP;
    _Float16 *vc = reinterpret_cast<_Float16 *>(a.vc) + (size_t)kvh * g.dvp * g.capp;
    const bool has_new = p < p0 + CHUNK;
    // what this workgroup reads from the cache is requested before anything else (the cache is padded to whole chunks:
    // positions beyond p exist and get no weight), unless it has to append first
    const int pi = tid >> 2, sub = tid & 3, ew = a.vdim <= 32 ? 32 : (a.vdim <= 64 ? 64 : (a.vdim <= 128 ? 128 : 256));
    const int e_first = tid % ew < a.vdim ? tid % ew : 0;
    half8 kf[NK], vf[CHUNK / 8];
    auto read_cache = [&]() {
#pragma unroll
        for (int c = 0; c < NK; c++) kf[c] = *reinterpret_cast<const half8 *>(kc + (size_t)(p0 + pi) * DP + (c * 4 + sub) * 8);
#pragma unroll
        for (int c = 0; c < CHUNK / 8; c++) vf[c] = *reinterpret_cast<const half8 *>(vc + (size_t)e_first * g.capp + p0 + c * 8);
    };
    if (!has_new) read_cache();
    const float temp = a.temp[p];
    for (int h = wave; h < rep; h += 4) {
        const float *q = g.q + (size_t)(kvh * rep + h) * a.dim;
        float ss = 0.f, qv[DP / 64];
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
            const int e = lane + i * 64;
            qv[i] = e < a.dim ? q[e] : 0.f;
            ss = fmaf(qv[i], qv[i], ss);
        }
        ss = axq_wave_sum(ss);
        const float f = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
            const int e = lane + i * 64;
            qs[h * DP + e] = e < a.dim ? qv[i] * f * a.qn[e] * temp : 0.f;
        }
    }
    if (has_new) { // append
        if (wave == (rep & 3)) {
            const float *k = g.k + (size_t)kvh * a.dim;
            float ss = 0.f;
            for (int e = lane; e < a.dim; e += 64) ss = fmaf(k[e], k[e], ss);
            ss = axq_wave_sum(ss);
            const float f = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
            for (int e = lane; e < a.dim; e += 64) kc[(size_t)p * DP + e] = to_half(k[e] * f * a.kn[e]);
        }
        if (wave == ((rep + 1) & 3)) {
            const float *v = g.v + (size_t)kvh * a.vdim;
            for (int e = lane; e < a.vdim; e += 64) vc[(size_t)e * g.capp + value_slot(p)] = to_half(v[e]);
        }
    }
    __syncthreads();
    if (has_new) read_cache();
    {
        const int j = p0 + pi, n = p - j < a.nt ? p - j : a.nt - 1;
        for (int h0 = 0; h0 < rep; h0 += 8) {
            float s[8];
#pragma unroll
            for (int i = 0; i < 8; i++) {
                s[i] = 0.f;
                if (h0 + i < rep) {
                    float t = 0.f;
#pragma unroll
                    for (int c = 0; c < NK; c++) {
                        const float *q = qs + (h0 + i) * DP + (c * 4 + sub) * 8;
                        const float4 qa = *reinterpret_cast<const float4 *>(q), qb = *reinterpret_cast<const float4 *>(q + 4);
                        t = fmaf(qa.x, (float)kf[c][0], t); t = fmaf(qa.y, (float)kf[c][1], t); t = fmaf(qa.z, (float)kf[c][2], t); t = fmaf(qa.w, (float)kf[c][3], t);
                        t = fmaf(qb.x, (float)kf[c][4], t); t = fmaf(qb.y, (float)kf[c][5], t); t = fmaf(qb.z, (float)kf[c][6], t); t = fmaf(qb.w, (float)kf[c][7], t);
                    }
                    s[i] = t;
                }
            }
#pragma unroll
            for (int i = 0; i < 8; i++) {
                float t = s[i];
                t += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, t), 0xB1, 0xf, 0xf, true));
                t += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, t), 0x4E, 0xf, 0xf, true));
                if (h0 + i < rep && sub == (i & 3))
                    ws[(h0 + i) * CHUNK + value_slot(pi)] = j <= p ? axq_sigmoid(fmaf(t, a.scale, a.bias[(size_t)(kvh * rep + h0 + i) * a.nt + n])) : 0.f;
            }
        }
    }
    __syncthreads();
    // value sums: thread = (element, head group), four heads at a time
    const int ng = 256 / ew, grp = tid / ew, e = tid % ew;
    if (e >= a.vdim) return;
    for (int h0 = grp; h0 < rep; h0 += 4 * ng) {
        float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < CHUNK / 8; c++) {
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int h = h0 + i * ng;
                if (h < rep) {
                    const float4 wa = *reinterpret_cast<const float4 *>(ws + h * CHUNK + c * 8), wb = *reinterpret_cast<const float4 *>(ws + h * CHUNK + c * 8 + 4);
                    float t = o[i];
                    t = fmaf(wa.x, (float)vf[c][0], t); t = fmaf(wa.y, (float)vf[c][1], t); t = fmaf(wa.z, (float)vf[c][2], t); t = fmaf(wa.w, (float)vf[c][3], t);
                    t = fmaf(wb.x, (float)vf[c][4], t); t = fmaf(wb.y, (float)vf[c][5], t); t = fmaf(wb.z, (float)vf[c][6], t); t = fmaf(wb.w, (float)vf[c][7], t);
                    o[i] = t;
                }
            }
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int h = h0 + i * ng;
            if (h < rep) part[((size_t)split * a.heads + kvh * rep + h) * a.vdim + e] = o[i];
        }
    }
}

// att[i] = sum over the splits of the newest position, in order; a workgroup takes 64 elements, its four waves every
// fourth split
__global__ void __launch_bounds__(256) token_combine_kernel(const float *part, const int32_t *pos, int n, float *att) {
    __shared__ float red[4][64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i = blockIdx.x * 64 + lane, splits = pos[0] / CHUNK + 1;
    float o = 0.f;
    if (i < n)
        for (int s = wave; s < splits; s += 4) o += part[(size_t)s * n + i];
    red[wave][lane] = o;
    __syncthreads();
    if (wave == 0 && i < n) att[i] = (red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]);
}

Args make_args(const axq_sig_attn &a, const float *q, const float *k, const float *v, int ldq, int ldk, int ldv, int m, int pos0,
               const int32_t *pos, void *qs) {
    Args g;
    g.a = a;
    g.q = q; g.k = k; g.v = v; g.ldq = ldq; g.ldk = ldk; g.ldv = ldv;
    g.m = m; g.pos0 = pos0; g.pos = pos;
    g.capp = pad_cap(a.cap); g.dp = pad_dim(a.dim); g.dvp = pad_dim(a.vdim);
    g.qs = qs;
    return g;
}

int check_shape(axq_ctx *ctx, const axq_sig_attn &a) {
    if (a.heads < 1 || a.kv_heads < 1 || a.heads % a.kv_heads || a.dim < 1 || a.vdim < 1 || a.dim > 256 || a.vdim > 256 || a.nt < 1 || a.cap < 1)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: attention of %d / %d heads, sizes %d and %d (at most 256)", a.heads,
                        a.kv_heads, a.dim, a.vdim);
    return AXQ_OK;
}

size_t f32_rows_lds(const axq_sig_attn &a) { return (size_t)(a.dim + 256 + (256 / a.vdim > 0 ? 256 / a.vdim : 1) * a.vdim) * sizeof(float); }

template <int KS, int DB>
int launch_mfma(axq_ctx *ctx, const Args &g, axq_rows_out out) {
    const int rep = g.a.heads / g.a.kv_heads, tiles = (g.m * rep + 127) / 128;
    constexpr size_t lds = (size_t)2 * (64 * KS * 16 + DB * 32 * 64) * sizeof(_Float16);
    static std::atomic<uint64_t> lds_allowed{0};
    int rc;
    if (lds > 48 * 1024 && (rc = axq_allow_lds(ctx, reinterpret_cast<const void *>(&rows_mfma_kernel<KS, DB>), lds_allowed, lds))) return rc;
    rows_mfma_kernel<KS, DB><<<dim3(g.a.kv_heads, tiles), 256, lds, ctx->stream>>>(g, out);
    return AXQ_OK;
}

template <int KS>
int launch_mfma_k(axq_ctx *ctx, const Args &g, axq_rows_out out) {
    if (g.dvp == 64) return launch_mfma<KS, 2>(ctx, g, out);
    if (g.dvp == 128) return launch_mfma<KS, 4>(ctx, g, out);
    return launch_mfma<KS, 8>(ctx, g, out);
}

template <int DP>
int launch_token(axq_ctx *ctx, const Args &g, float *part) {
    const size_t lds = (size_t)(g.a.heads / g.a.kv_heads) * (DP + CHUNK) * sizeof(float);
    static std::atomic<uint64_t> lds_allowed{0};
    int rc;
    if (lds > 128 * 1024)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: %d query heads per KV head of size %d", g.a.heads / g.a.kv_heads, g.a.dim);
    if (lds > 48 * 1024 && (rc = axq_allow_lds(ctx, reinterpret_cast<const void *>(&token_partial_kernel<DP>), lds_allowed, 128 * 1024))) return rc;
    token_partial_kernel<DP><<<dim3(g.a.kv_heads, g.capp / CHUNK), 256, lds, ctx->stream>>>(g, part);
    return AXQ_OK;
}

} // namespace

size_t axq_sig_attn_k_bytes(const axq_sig_attn &a) {
    return a.f32 ? (size_t)a.kv_heads * a.cap * a.dim * 4 : (size_t)a.kv_heads * pad_cap(a.cap) * pad_dim(a.dim) * 2;
}
size_t axq_sig_attn_v_bytes(const axq_sig_attn &a) {
    return a.f32 ? (size_t)a.kv_heads * a.cap * a.vdim * 4 : (size_t)a.kv_heads * pad_cap(a.cap) * pad_dim(a.vdim) * 2;
}
size_t axq_sig_attn_q_bytes(const axq_sig_attn &a, int m) { return (size_t)m * a.heads * pad_dim(a.dim) * (a.f32 ? 4 : 2); }
size_t axq_sig_attn_part_bytes(const axq_sig_attn &a) { return (size_t)(pad_cap(a.cap) / CHUNK) * a.heads * a.vdim * 4; }

int axq_sig_attn_rows(axq_ctx *ctx, const axq_sig_attn &a, const float *q, const float *k, const float *v, int ldq, int ldk, int ldv, int m,
                      int pos0, void *qscratch, axq_rows_out out) {
    int rc;
    if ((rc = check_shape(ctx, a))) return rc;
    if (m < 1 || pos0 < 0 || pos0 + m > a.cap)
        return axq_fail(ctx, AXQ_ERR_OVERFLOW, "Numerical overflow during quantization: positions %d .. %d beyond the cache of %d", pos0, pos0 + m, a.cap);
    const Args g = make_args(a, q, k, v, ldq, ldk, ldv, m, pos0, nullptr, qscratch);
    if (a.f32) {
        prep_kernel<true><<<dim3(a.heads + 2 * a.kv_heads, m), 64, 0, ctx->stream>>>(g);
        rows_f32_kernel<<<dim3(a.heads, m), 256, f32_rows_lds(a), ctx->stream>>>(g, out);
    } else {
        prep_kernel<false><<<dim3(a.heads + a.kv_heads, m), 64, 0, ctx->stream>>>(g);
        append_values_kernel<<<dim3((m + 31) / 32, (a.vdim + 31) / 32, a.kv_heads), 256, 0, ctx->stream>>>(g);
        if ((rc = g.dp == 64 ? launch_mfma_k<4>(ctx, g, out) : (g.dp == 128 ? launch_mfma_k<8>(ctx, g, out) : launch_mfma_k<16>(ctx, g, out)))) return rc;
    }
    AXQ_LAUNCH_CHECK(ctx, "sigmoid attention of rows");
    return axq_rows_zero_tail(ctx, m, a.heads * a.vdim, out);
}

int axq_sig_attn_token(axq_ctx *ctx, const axq_sig_attn &a, const float *q, const float *k, const float *v, const int32_t *pos, void *qscratch,
                       float *part, float *att) {
    int rc;
    if ((rc = check_shape(ctx, a))) return rc;
    const Args g = make_args(a, q, k, v, 0, 0, 0, 1, 0, pos, qscratch);
    if (a.f32) {
        prep_kernel<true><<<dim3(a.heads + 2 * a.kv_heads, 1), 64, 0, ctx->stream>>>(g);
        axq_rows_out out = {att, a.heads * a.vdim, true};
        rows_f32_kernel<<<dim3(a.heads, 1), 256, f32_rows_lds(a), ctx->stream>>>(g, out);
    } else {
        const int n = a.heads * a.vdim;
        if ((rc = g.dp == 64 ? launch_token<64>(ctx, g, part) : (g.dp == 128 ? launch_token<128>(ctx, g, part) : launch_token<256>(ctx, g, part)))) return rc;
        token_combine_kernel<<<(n + 63) / 64, 256, 0, ctx->stream>>>(part, pos, n, att);
    }
    AXQ_LAUNCH_CHECK(ctx, "sigmoid attention of a token");
    return AXQ_OK;
}
