// Causal softmax attention over a sliding window of tokens and, where asked for, the means of blocks of older tokens:
// with s = max(0, p - window + 1), position p sees the tokens s .. p and the first s / pool blocks of `pool` tokens, each as one
// key and one value, the means of the cached ones (what lies between the last whole block and s is not seen).  Queries and keys may be rotated in part (neighbouring dimensions), values may
// be the keys before rotation, each head's result may be gated.
//
// The blocks' keys and values are a second cache of the same layout (axq_attn_tiles.h); all kernels walk the blocks first and
// the window after them with one running maximum.  A block's means are taken from the cache when its last token is
// appended, so they do not depend on how the tokens came; no position sees a block before that.
#include "axq_attn_tiles.h"

namespace {

struct Args {
    axq_soft_attn a;
    const float *q, *k, *v, *gate;
    int ldq, ldk, ldv;
    int m, pos0;
    const int32_t *pos;      // != NULL: one row at *pos
    int capp, cpp, dp, dvp;  // f16 caches: padded positions and blocks, padded head sizes
    int cap_blocks;
    void *qs;                // prepared queries: f16 [m][heads][dp] or f32 [m][heads][dim]
};

__device__ inline int first_token(const axq_soft_attn &a, int p) { return p - a.window + 1 > 0 ? p - a.window + 1 : 0; }
__device__ inline int seen_blocks(const axq_soft_attn &a, int p) { return a.pool > 0 && p - a.window + 1 > 0 ? (p - a.window + 1) / a.pool : 0; }

// Element e of a head's vector x at position p, rotated where rotation reaches.
__device__ inline float rotated(const axq_soft_attn &a, const float *x, int e, int p) {
    const float v = x[e];
    if (e >= a.rot_dims) return v;
    const size_t i = (size_t)p * (a.rot_dims >> 1) + (e >> 1);
    const float c = a.rc[i], s = a.rs[i], w = x[e ^ 1];
    return (e & 1) ? fmaf(v, c, w * s) : fmaf(v, c, -(w * s));
}

// grid (heads + kv_heads (+ kv_heads of values in f32) in fours, rows), a wave each: rotated queries, keys into the cache
template <bool F32>
__global__ void __launch_bounds__(256) prep_kernel(Args g) {
    const axq_soft_attn &a = g.a;
    const int t = blockIdx.y, lane = threadIdx.x & 63, p = g.pos ? g.pos[0] : g.pos0 + t;
    int h = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (h >= a.heads + (F32 ? 2 : 1) * a.kv_heads) return;
    if (h < a.heads) {
        const float *q = g.q + (size_t)t * g.ldq + (size_t)h * a.dim;
        if (F32) {
            float *o = reinterpret_cast<float *>(g.qs) + ((size_t)t * a.heads + h) * a.dim;
            for (int e = lane; e < a.dim; e += 64) o[e] = rotated(a, q, e, p);
        } else {
            _Float16 *o = reinterpret_cast<_Float16 *>(g.qs) + ((size_t)t * a.heads + h) * g.dp;
            for (int e = lane; e < g.dp; e += 64) o[e] = e < a.dim ? to_half(rotated(a, q, e, p)) : (_Float16)0.f;
        }
        return;
    }
    h -= a.heads;
    if (h < a.kv_heads) {
        const float *k = g.k + (size_t)t * g.ldk + (size_t)h * a.dim;
        if (F32) {
            float *o = reinterpret_cast<float *>(a.kc) + ((size_t)h * a.cap + p) * a.dim;
            for (int e = lane; e < a.dim; e += 64) o[e] = rotated(a, k, e, p);
        } else {
            _Float16 *o = reinterpret_cast<_Float16 *>(a.kc) + ((size_t)h * g.capp + p) * g.dp;
            for (int e = lane; e < a.dim; e += 64) o[e] = to_half(rotated(a, k, e, p)); // the padding stays zero
        }
        return;
    }
    h -= a.kv_heads;
    const float *v = g.v + (size_t)t * g.ldv + (size_t)h * a.vdim;
    float *o = reinterpret_cast<float *>(a.vc) + ((size_t)h * a.cap + p) * a.vdim;
    for (int e = lane; e < a.vdim; e += 64) o[e] = v[e];
}

__global__ void __launch_bounds__(256) append_values_kernel(Args g) { append_values(g.v, g.ldv, g.a.vdim, g.m, g.pos0, g.a.vc, g.dvp, g.capp); }

// The means of block b for kv head h, by the threads tid, tid + n, ... of n.
template <bool F32>
__device__ void pool_block(const Args &g, int h, int b, int tid, int n) {
    const axq_soft_attn &a = g.a;
    const float inv = 1.0f / (float)a.pool;
    const size_t p0 = (size_t)b * a.pool;
    for (int i = tid; i < a.dim + a.vdim; i += n) {
        const bool key = i < a.dim;
        const int e = key ? i : i - a.dim;
        float s = 0.f;
        if (F32) {
            const int d = key ? a.dim : a.vdim;
            const float *x = reinterpret_cast<const float *>(key ? a.kc : a.vc) + ((size_t)h * a.cap + p0) * d + e;
#pragma unroll 16
            for (int j = 0; j < a.pool; j++) s += x[(size_t)j * d];
            reinterpret_cast<float *>(key ? a.pkc : a.pvc)[((size_t)h * g.cap_blocks + b) * d + e] = s * inv;
        } else if (key) {
            const _Float16 *x = reinterpret_cast<const _Float16 *>(a.kc) + ((size_t)h * g.capp + p0) * g.dp + e;
#pragma unroll 16
            for (int j = 0; j < a.pool; j++) s += (float)x[(size_t)j * g.dp];
            reinterpret_cast<_Float16 *>(a.pkc)[((size_t)h * g.cpp + b) * g.dp + e] = (_Float16)(s * inv);
        } else {
            const _Float16 *x = reinterpret_cast<const _Float16 *>(a.vc) + ((size_t)h * g.dvp + e) * g.capp;
#pragma unroll 16
            for (int j = 0; j < a.pool; j++) s += (float)x[value_slot((int)p0 + j)];
            reinterpret_cast<_Float16 *>(a.pvc)[((size_t)h * g.dvp + e) * g.cpp + value_slot(b)] = (_Float16)(s * inv);
        }
    }
}

// grid (kv heads, blocks that end within the rows)
template <bool F32>
__global__ void __launch_bounds__(256) pool_kernel(Args g) {
    int b;
    if (g.pos) {
        const int n = g.pos[0] + 1;
        if (n % g.a.pool != 0) return;
        b = n / g.a.pool - 1;
    } else {
        b = g.pos0 / g.a.pool + blockIdx.y;
    }
    pool_block<F32>(g, blockIdx.x, b, threadIdx.x, 256);
}

// Rows against the f32 caches: grid (heads, rows).  256 keys at a time: scores by thread, then the value sum by element.
__global__ void __launch_bounds__(256) rows_f32_kernel(Args g, axq_rows_out out) {
    extern __shared__ float sm[];
    const axq_soft_attn &a = g.a;
    const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, p = g.pos ? g.pos[0] : g.pos0 + t;
    const int kvh = h / (a.heads / a.kv_heads), ng = 256 / a.vdim > 0 ? 256 / a.vdim : 1;
    float *qs = sm, *w = qs + a.dim, *stat = w + 256, *red = stat + 8; // stat: a value per wave; red [ng][vdim]
    const float *q = reinterpret_cast<const float *>(g.qs) + ((size_t)t * a.heads + h) * a.dim;
    const float *kc = reinterpret_cast<const float *>(a.kc) + (size_t)kvh * a.cap * a.dim;
    const float *vc = reinterpret_cast<const float *>(a.vc) + (size_t)kvh * a.cap * a.vdim;
    const float *pkc = reinterpret_cast<const float *>(a.pkc) + (size_t)kvh * g.cap_blocks * a.dim;
    const float *pvc = reinterpret_cast<const float *>(a.pvc) + (size_t)kvh * g.cap_blocks * a.vdim;
    const int nb = seen_blocks(a, p), lo = first_token(a, p), n = nb + p - lo + 1; // keys: blocks 0 .. nb - 1, then tokens lo .. p
    for (int e = tid; e < a.dim; e += 256) qs[e] = q[e];
    for (int e = tid; e < ng * a.vdim; e += 256) red[e] = 0.f;
    float top = -1e30f, sum = 0.f;
    __syncthreads();
    for (int j0 = 0; j0 < n; j0 += 256) {
        const int j = j0 + tid;
        float s = -INFINITY;
        if (j < n) {
            const float *k = j < nb ? pkc + (size_t)j * a.dim : kc + (size_t)(lo + j - nb) * a.dim;
            s = 0.f;
            for (int e = 0; e < a.dim; e++) s = fmaf(qs[e], k[e], s);
            s *= a.scale;
        }
        float mx = s;
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) mx = fmaxf(mx, __shfl_xor(mx, d));
        if ((tid & 63) == 0) stat[tid >> 6] = mx;
        __syncthreads();
        const float next = fmaxf(fmaxf(fmaxf(stat[0], stat[1]), fmaxf(stat[2], stat[3])), top), f = expf(top - next);
        const float wt = expf(s - next), ws = axq_wave_sum(wt);
        w[tid] = wt;
        if ((tid & 63) == 0) stat[4 + (tid >> 6)] = ws;
        __syncthreads();
        sum = fmaf(sum, f, (stat[4] + stat[5]) + (stat[6] + stat[7]));
        top = next;
        const int nj = n - j0 < 256 ? n - j0 : 256;
        for (int i = tid; i < ng * a.vdim; i += 256) {
            const int e = i % a.vdim, grp = i / a.vdim;
            float o = red[i] * f;
            for (int jj = grp; jj < nj; jj += ng) {
                const int x = j0 + jj;
                o = fmaf(w[jj], x < nb ? pvc[(size_t)x * a.vdim + e] : vc[(size_t)(lo + x - nb) * a.vdim + e], o);
            }
            red[i] = o;
        }
        __syncthreads();
    }
    const float inv = (g.gate ? g.gate[(size_t)t * a.heads + h] : 1.0f) / sum;
    for (int e = tid; e < a.vdim; e += 256) {
        float o = 0.f;
        for (int grp = 0; grp < ng; grp++) o += red[grp * a.vdim + e];
        o *= inv;
        if (out.f32) reinterpret_cast<float *>(out.x)[(size_t)t * out.ldx + (size_t)h * a.vdim + e] = o;
        else reinterpret_cast<uint16_t *>(out.x)[(size_t)t * out.ldx + (size_t)h * a.vdim + e] = axq_to_bf16(o);
    }
}

// Rows against the f16 caches on the matrix pipe.  A wave takes 32 "virtual queries" (row, query head of the group),
// which are lanes (column lane % 32) all the way through:
//   S^T = K Q^T (32 keys x 32 queries), A = key rows, B = queries;
//   P^T = exp2(S - running maximum of the query) as f16: the accumulator of a lane holds keys 8 i + 4 (lane / 32) + 0..3, and
//         the second product sums over the keys in that very order (value_slot), so P needs no exchange of lanes;
//   O^T += V^T P^T, A = rows of the transposed values; a new maximum scales a lane's own accumulators.
// The four waves of a workgroup walk the same keys, 64 at a time (the blocks any of its queries sees, then the tokens), through
// LDS: two stages, filled straight from memory; the 16-byte pieces of a row are exchanged by row % 8 so that operand reads use
// all banks.  Workgroups with the longest ranges start first.
template <int KS, int DB>
__global__ void __launch_bounds__(256, KS + DB > 20 ? 1 : 2) rows_mfma_kernel(Args g, axq_rows_out out) {
    constexpr int DP = KS * 16, DVP = DB * 32, KC = DP / 8; // KC: 16-byte pieces of a key row
    constexpr int KH = 64 * DP, STAGE = KH + DVP * 64;       // halfs of a key tile, of a stage
    extern __shared__ __attribute__((aligned(16))) _Float16 tiles[];
    const axq_soft_attn &a = g.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 31, lh = lane >> 5;
    const int kvh = blockIdx.x, rep = a.heads / a.kv_heads, wg = (int)gridDim.y - 1 - (int)blockIdx.y;
    const int total = g.m * rep, vq0 = (wg * 4 + wave) * 32;
    const int vq = vq0 + li, vqc = vq < total ? vq : total - 1;
    const int row = vqc / rep, h = kvh * rep + vqc % rep, p = g.pos0 + row;
    const int last = vq0 + 31 < total ? vq0 + 31 : total - 1, p_min = g.pos0 + (vq0 < total ? vq0 : total - 1) / rep, p_max = g.pos0 + last / rep;
    const int wg_last = wg * 128 + 127 < total ? wg * 128 + 127 : total - 1, wg_min = g.pos0 + wg * 128 / rep, wg_max = g.pos0 + wg_last / rep;
    const int nb = seen_blocks(a, p), lo = first_token(a, p);                  // this lane's query
    const int nb_min = seen_blocks(a, p_min), nb_max = seen_blocks(a, p_max), lo_min = first_token(a, p_min), lo_max = first_token(a, p_max); // this wave's
    const int ptiles = (seen_blocks(a, wg_max) + 63) >> 6, tile0 = first_token(a, wg_min) >> 6, ntiles = ptiles + (wg_max >> 6) - tile0 + 1;
    const _Float16 *gk[DP / 32], *gv[DB];
    auto aim = [&](const void *kc, const void *vc, int cap) { // at a cache's first tile
        const _Float16 *k = reinterpret_cast<const _Float16 *>(kc) + (size_t)kvh * cap * DP;
        const _Float16 *v = reinterpret_cast<const _Float16 *>(vc) + (size_t)kvh * DVP * cap;
#pragma unroll
        for (int i = 0; i < DP / 32; i++) {
            const int idx = (i * 4 + wave) * 64 + lane, r = idx / KC, c = (idx % KC) ^ (r & 7);
            gk[i] = k + (size_t)r * DP + c * 8;
        }
#pragma unroll
        for (int i = 0; i < DB; i++) {
            const int idx = (i * 4 + wave) * 64 + lane, r = idx >> 3, c = (idx & 7) ^ (r & 7);
            gv[i] = v + (size_t)r * cap + c * 8;
        }
    };
    auto fetch = [&](int stage, int tile) { // both caches are padded to whole tiles
        if (tile == ptiles) aim(a.kc, a.vc, g.capp);
        const int j0 = (tile < ptiles ? tile : tile0 + tile - ptiles) * 64;
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
    const float scale = a.scale * LOG2E;
    float top = -1e30f, sum = 0.f; // sum: of this half wave's keys, times PSCALE
    if (ptiles > 0) aim(a.pkc, a.pvc, g.cpp);
    fetch(0, 0);
    for (int tile = 0; tile < ntiles; tile++) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); // this tile is in LDS ...
        __syncthreads();                                  // ... of every wave, and nobody reads the other stage any more
        if (tile + 1 < ntiles) fetch((tile + 1) & 1, tile + 1);
        const bool blocks = tile < ptiles;
        const int t0 = (blocks ? tile : tile0 + tile - ptiles) * 64;
        const _Float16 *lk = tiles + (tile & 1) * STAGE, *lv = lk + KH;
#pragma unroll
        for (int sub = 0; sub < 2; sub++) {
            const int j0 = t0 + sub * 32;
            if (blocks ? j0 >= nb_max : j0 > p_max || j0 + 31 < lo_min) continue; // nobody in the wave sees any of it
            f32x16 S;
#pragma unroll
            for (int r = 0; r < 16; r++) S[r] = 0.f;
#pragma unroll
            for (int ks = 0; ks < KS; ks++) {
                const half8 kf = *reinterpret_cast<const half8 *>(lk + (sub * 32 + li) * DP + (((ks * 2 + lh) ^ (li & 7)) << 3));
                S = __builtin_amdgcn_mfma_f32_32x32x16_f16(kf, qf[ks], S, 0, 0, 0);
            }
            if (blocks ? j0 + 32 > nb_min : j0 + 31 > p_min || j0 < lo_max) { // somebody does not see all of it
                const int first = blocks ? 0 : lo, end = blocks ? nb : p + 1;
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    const int j = j0 + acc_row(r, lane);
                    if (j < first || j >= end) S[r] = -INFINITY;
                }
            }
            float mx = S[0];
#pragma unroll
            for (int r = 1; r < 16; r++) mx = fmaxf(mx, S[r]);
            mx = fmaxf(mx, __shfl_xor(mx, 32)) * scale;
            if (__builtin_amdgcn_ballot_w64(mx > top)) { // a scale below zero would need the smallest: refused at creation
                const float next = fmaxf(mx, top), f = __builtin_amdgcn_exp2f(top - next);
                top = next;
                sum *= f;
#pragma unroll
                for (int db = 0; db < DB; db++)
#pragma unroll
                    for (int r = 0; r < 16; r++) O[db][r] *= f;
            }
            half8 pf[2];
            const float off = 15.0f - top; // log2 of PSCALE
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const float w = __builtin_amdgcn_exp2f(fmaf(S[r], scale, off));
                sum += w;
                pf[r >> 3][r & 7] = (_Float16)w;
            }
#pragma unroll
            for (int ks = 0; ks < 2; ks++)
#pragma unroll
                for (int db = 0; db < DB; db++) {
                    const half8 vf = *reinterpret_cast<const half8 *>(lv + (db * 32 + li) * 64 + (((sub * 4 + ks * 2 + lh) ^ (li & 7)) << 3));
                    O[db] = __builtin_amdgcn_mfma_f32_32x32x16_f16(vf, pf[ks], O[db], 0, 0, 0);
                }
        }
    }
    sum += __shfl_xor(sum, 32);
    if (vq >= total) return;
    const float inv = (g.gate ? g.gate[(size_t)row * a.heads + h] : 1.0f) / sum;
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int e = db * 32 + acc_row(r, lane);
            if (e < a.vdim) {
                const float o = O[db][r] * inv;
                const size_t i = (size_t)row * out.ldx + (size_t)h * a.vdim + e;
                if (out.f32) reinterpret_cast<float *>(out.x)[i] = o;
                else reinterpret_cast<uint16_t *>(out.x)[i] = axq_to_bf16(o);
            }
        }
}

// One token, f16 caches: workgroup (kv head, split) takes 64 keys for all query heads of the group: the splits below
// cpp / 64 blocks 64 split .., the others the window's tokens, from the 64 that hold its first one on.  The workgroup whose
// range holds the newest position appends that position's key and value first, and the means of a block that it completes (no
// workgroup of this step reads those).  Workgroups without keys leave at once (the grid is sized for the whole window so that the
// launch can sit in a graph).  A split leaves, per head, its value sum, its largest score and its sum of weights.
struct Split { int base, first, end, blocks; }; // keys first .. end - 1 of base .. base + 63
__device__ inline bool split_of(const axq_soft_attn &a, int psplits, int split, int p, Split &s) {
    const int lo = first_token(a, p);
    s.blocks = split < psplits;
    s.base = s.blocks ? split * CHUNK : ((lo / CHUNK) + split - psplits) * CHUNK;
    s.first = s.blocks ? 0 : lo;
    s.end = s.blocks ? seen_blocks(a, p) : p + 1;
    return s.base < s.end;
}

template <int DP>
__global__ void __launch_bounds__(256) token_partial_kernel(Args g, float *part) {
    extern __shared__ __attribute__((aligned(16))) float sm2[];
    constexpr int NK = DP / 32; // 16-byte pieces of a key per lane: four lanes take a position's pieces in turn
    constexpr float LOG2E = 1.4426950408889634f;
    const axq_soft_attn &a = g.a;
    const int kvh = blockIdx.x, split = blockIdx.y, p = g.pos[0], psplits = g.cpp / CHUNK;
    Split sp;
    if (!split_of(a, psplits, split, p, sp)) return;
    const int rep = a.heads / a.kv_heads, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, p0 = sp.base, cap = sp.blocks ? g.cpp : g.capp;
    float *qs = sm2, *ws = qs + (size_t)rep * DP; // [rep][DP], [rep][CHUNK] (columns in value_slot order)
    _Float16 *kc = reinterpret_cast<_Float16 *>(sp.blocks ? a.pkc : a.kc) + (size_t)kvh * cap * DP;
    _Float16 *vc = reinterpret_cast<_Float16 *>(sp.blocks ? a.pvc : a.vc) + (size_t)kvh * g.dvp * cap;
    const bool has_new = !sp.blocks && p < p0 + CHUNK;
    // what this workgroup reads from the cache is requested before anything else (the caches are padded to whole chunks: keys
    // that are not seen exist and get no weight), unless it has to append first
    const int pi = tid >> 2, sub = tid & 3, ew = a.vdim <= 32 ? 32 : (a.vdim <= 64 ? 64 : (a.vdim <= 128 ? 128 : 256));
    const int e_first = tid % ew < a.vdim ? tid % ew : 0;
    half8 kf[NK], vf[CHUNK / 8];
    auto read_cache = [&]() {
#pragma unroll
        for (int c = 0; c < NK; c++) kf[c] = *reinterpret_cast<const half8 *>(kc + (size_t)(p0 + pi) * DP + (c * 4 + sub) * 8);
#pragma unroll
        for (int c = 0; c < CHUNK / 8; c++) vf[c] = *reinterpret_cast<const half8 *>(vc + (size_t)e_first * cap + p0 + c * 8);
    };
    if (!has_new) read_cache();
    for (int h = wave; h < rep; h += 4) {
        const float *q = g.q + (size_t)(kvh * rep + h) * a.dim;
        for (int e = lane; e < DP; e += 64) qs[h * DP + e] = e < a.dim ? rotated(a, q, e, p) : 0.f;
    }
    if (has_new) { // append
        if (wave == (rep & 3)) {
            const float *k = g.k + (size_t)kvh * a.dim;
            for (int e = lane; e < a.dim; e += 64) kc[(size_t)p * DP + e] = to_half(rotated(a, k, e, p));
        }
        if (wave == ((rep + 1) & 3)) {
            const float *v = g.v + (size_t)kvh * a.vdim;
            for (int e = lane; e < a.vdim; e += 64) vc[(size_t)e * cap + value_slot(p)] = to_half(v[e]);
        }
    }
    __syncthreads();
    if (has_new) {
        read_cache();
        if (a.pool > 0 && (p + 1) % a.pool == 0) pool_block<false>(g, kvh, (p + 1) / a.pool - 1, tid, 256);
    }
    {
        const int j = p0 + pi;
        const bool seen = j >= sp.first && j < sp.end;
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
                if (h0 + i < rep && sub == (i & 3)) ws[(h0 + i) * CHUNK + value_slot(pi)] = seen ? t * (a.scale * LOG2E) : -INFINITY;
            }
        }
    }
    __syncthreads();
    const int ldp = a.vdim + 2;
    for (int h = wave; h < rep; h += 4) { // scores of a head -> weights under the split's maximum
        const float s = ws[h * CHUNK + lane];
        float mx = s;
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) mx = fmaxf(mx, __shfl_xor(mx, d));
        const float w = __builtin_amdgcn_exp2f(s - mx); // a split has keys, so mx is finite
        const float sum = axq_wave_sum(w);
        ws[h * CHUNK + lane] = w;
        if (lane == 0) {
            float *o = part + ((size_t)split * a.heads + kvh * rep + h) * ldp + a.vdim;
            o[0] = mx;
            o[1] = sum;
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
            if (h < rep) part[((size_t)split * a.heads + kvh * rep + h) * ldp + e] = o[i];
        }
    }
}

// The splits of the newest position put together: workgroup (head, 64 elements), its four waves every fourth split.
__global__ void __launch_bounds__(256) token_combine_kernel(Args g, const float *part, float *att) {
    __shared__ float red[4][64];
    const axq_soft_attn &a = g.a;
    const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, e = blockIdx.y * 64 + lane, p = g.pos[0], ldp = a.vdim + 2;
    const int psplits = g.cpp / CHUNK, np = (seen_blocks(a, p) + CHUNK - 1) / CHUNK, n = np + p / CHUNK - first_token(a, p) / CHUNK + 1;
    auto at = [&](int i) { return part + ((size_t)(i < np ? i : psplits + i - np) * a.heads + h) * ldp; };
    float mx = -1e30f;
    for (int i = lane; i < n; i += 64) mx = fmaxf(mx, at(i)[a.vdim]);
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) mx = fmaxf(mx, __shfl_xor(mx, d));
    float sum = 0.f;
    for (int i = lane; i < n; i += 64) sum = fmaf(at(i)[a.vdim + 1], __builtin_amdgcn_exp2f(at(i)[a.vdim] - mx), sum);
    sum = axq_wave_sum(sum);
    float o = 0.f;
    if (e < a.vdim)
        for (int i = wave; i < n; i += 4) o = fmaf(at(i)[e], __builtin_amdgcn_exp2f(at(i)[a.vdim] - mx), o);
    red[wave][lane] = o;
    __syncthreads();
    if (wave == 0 && e < a.vdim)
        att[(size_t)h * a.vdim + e] = ((red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane])) * ((g.gate ? g.gate[h] : 1.0f) / sum);
}

inline int blocks_of(const axq_soft_attn &a) { return a.pool > 0 ? a.cap / a.pool : 0; }
// splits of a decode step: of the blocks, of the window's tokens
inline int pool_splits(const axq_soft_attn &a) { return pad_cap(blocks_of(a)) / CHUNK; }
inline int token_splits(const axq_soft_attn &a) {
    const int all = pad_cap(a.cap) / CHUNK, win = (a.window < a.cap ? a.window : a.cap) / CHUNK + 2;
    return win < all ? win : all;
}

Args make_args(const axq_soft_attn &a, const float *q, const float *k, const float *v, const float *gate, int ldq, int ldk, int ldv, int m,
               int pos0, const int32_t *pos, void *qs) {
    Args g;
    g.a = a;
    g.q = q; g.k = k; g.v = v; g.gate = gate; g.ldq = ldq; g.ldk = ldk; g.ldv = ldv;
    g.m = m; g.pos0 = pos0; g.pos = pos;
    g.cap_blocks = blocks_of(a);
    g.capp = pad_cap(a.cap); g.cpp = pad_cap(g.cap_blocks); g.dp = pad_dim(a.dim); g.dvp = pad_dim(a.vdim);
    g.qs = qs;
    return g;
}

int check_shape(axq_ctx *ctx, const axq_soft_attn &a) {
    if (a.heads < 1 || a.kv_heads < 1 || a.heads % a.kv_heads || a.dim < 1 || a.vdim < 1 || a.dim > 256 || a.vdim > 256 || a.cap < 1 ||
        a.window < 1 || a.pool < 0 || a.rot_dims < 0 || a.rot_dims > a.dim || a.rot_dims % 2 || !(a.scale > 0.f))
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: attention of %d / %d heads, sizes %d and %d (at most 256), window %d, blocks of %d, %d "
                        "rotated", a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.pool, a.rot_dims);
    return AXQ_OK;
}

size_t f32_rows_lds(const axq_soft_attn &a) { return (size_t)(a.dim + 264 + (256 / a.vdim > 0 ? 256 / a.vdim : 1) * a.vdim) * sizeof(float); }

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
    token_partial_kernel<DP><<<dim3(g.a.kv_heads, pool_splits(g.a) + token_splits(g.a)), 256, lds, ctx->stream>>>(g, part);
    return AXQ_OK;
}

template <bool F32>
void launch_pool(axq_ctx *ctx, const Args &g) {
    if (g.a.pool < 1 || g.cap_blocks < 1) return;
    const int n = g.pos ? 1 : (g.pos0 + g.m) / g.a.pool - g.pos0 / g.a.pool;
    if (n > 0) pool_kernel<F32><<<dim3(g.a.kv_heads, n), 256, 0, ctx->stream>>>(g);
}

} // namespace

size_t axq_soft_attn_k_bytes(const axq_soft_attn &a) {
    return a.f32 ? (size_t)a.kv_heads * a.cap * a.dim * 4 : (size_t)a.kv_heads * pad_cap(a.cap) * pad_dim(a.dim) * 2;
}
size_t axq_soft_attn_v_bytes(const axq_soft_attn &a) {
    return a.f32 ? (size_t)a.kv_heads * a.cap * a.vdim * 4 : (size_t)a.kv_heads * pad_cap(a.cap) * pad_dim(a.vdim) * 2;
}
size_t axq_soft_attn_pk_bytes(const axq_soft_attn &a) {
    return a.f32 ? (size_t)a.kv_heads * blocks_of(a) * a.dim * 4 : (size_t)a.kv_heads * pad_cap(blocks_of(a)) * pad_dim(a.dim) * 2;
}
size_t axq_soft_attn_pv_bytes(const axq_soft_attn &a) {
    return a.f32 ? (size_t)a.kv_heads * blocks_of(a) * a.vdim * 4 : (size_t)a.kv_heads * pad_cap(blocks_of(a)) * pad_dim(a.vdim) * 2;
}
size_t axq_soft_attn_q_bytes(const axq_soft_attn &a, int m) { return (size_t)m * a.heads * pad_dim(a.dim) * (a.f32 ? 4 : 2); }
size_t axq_soft_attn_part_bytes(const axq_soft_attn &a) { return (size_t)(pool_splits(a) + token_splits(a)) * a.heads * (a.vdim + 2) * 4; }

int axq_soft_attn_rows(axq_ctx *ctx, const axq_soft_attn &a, const float *q, const float *k, const float *v, int ldq, int ldk, int ldv,
                       const float *gate, int m, int pos0, void *qscratch, axq_rows_out out) {
    int rc;
    if ((rc = check_shape(ctx, a))) return rc;
    if (m < 1 || pos0 < 0 || pos0 + m > a.cap)
        return axq_fail(ctx, AXQ_ERR_OVERFLOW, "Numerical overflow during quantization: positions %d .. %d beyond the cache of %d", pos0, pos0 + m, a.cap);
    const Args g = make_args(a, q, k, v, gate, ldq, ldk, ldv, m, pos0, nullptr, qscratch);
    if (a.f32) {
        prep_kernel<true><<<dim3((a.heads + 2 * a.kv_heads + 3) / 4, m), 256, 0, ctx->stream>>>(g);
        launch_pool<true>(ctx, g);
        rows_f32_kernel<<<dim3(a.heads, m), 256, f32_rows_lds(a), ctx->stream>>>(g, out);
    } else {
        prep_kernel<false><<<dim3((a.heads + a.kv_heads + 3) / 4, m), 256, 0, ctx->stream>>>(g);
        append_values_kernel<<<dim3((m + 31) / 32, (a.vdim + 31) / 32, a.kv_heads), 256, 0, ctx->stream>>>(g);
        launch_pool<false>(ctx, g);
        if ((rc = g.dp == 64 ? launch_mfma_k<4>(ctx, g, out) : (g.dp == 128 ? launch_mfma_k<8>(ctx, g, out) : launch_mfma_k<16>(ctx, g, out)))) return rc;
    }
    AXQ_LAUNCH_CHECK(ctx, "softmax attention of rows");
    return axq_rows_zero_tail(ctx, m, a.heads * a.vdim, out);
}

int axq_soft_attn_token(axq_ctx *ctx, const axq_soft_attn &a, const float *q, const float *k, const float *v, const float *gate,
                        const int32_t *pos, void *qscratch, float *part, float *att) {
    int rc;
    if ((rc = check_shape(ctx, a))) return rc;
    const Args g = make_args(a, q, k, v, gate, 0, 0, 0, 1, 0, pos, qscratch);
    if (a.f32) {
        prep_kernel<true><<<dim3((a.heads + 2 * a.kv_heads + 3) / 4, 1), 256, 0, ctx->stream>>>(g);
        launch_pool<true>(ctx, g);
        axq_rows_out out = {att, a.heads * a.vdim, true};
        rows_f32_kernel<<<dim3(a.heads, 1), 256, f32_rows_lds(a), ctx->stream>>>(g, out);
    } else {
        if ((rc = g.dp == 64 ? launch_token<64>(ctx, g, part) : (g.dp == 128 ? launch_token<128>(ctx, g, part) : launch_token<256>(ctx, g, part)))) return rc;
        token_combine_kernel<<<dim3(a.heads, (a.vdim + 63) / 64), 256, 0, ctx->stream>>>(g, part, att);
    }
    AXQ_LAUNCH_CHECK(ctx, "softmax attention of a token");
    return AXQ_OK;
}
