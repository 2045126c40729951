// Products with bfloat16 weights: the GEMV of a decode step (input transforms, activations and residual adds ride in
// it) and the GEMM of many rows (bf16 rows on the matrix pipe, or f32 rows in true 32-bit), both over several weights
// per launch; and the row operations of a prompt around them.
#include "axq_dense.h"

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x4_any __attribute__((ext_vector_type(4), aligned(4))); // at any float's address
typedef const __attribute__((address_space(1))) void gbl_void;
typedef __attribute__((address_space(3))) void lds_void;

__device__ inline float tanh_norm(float x, float alpha, float w, float b) { return tanhf(alpha * x) * w + b; }

// ---------------------------------------------------------------------------------------------------------------------
// GEMV.  A workgroup (eight waves) stages f(x) in LDS once per distinct input and walks a contiguous range of row blocks
// (8 R rows, R per wave); a lane's step is 16 bytes (8 weights) of each of its R rows, U steps make an item.  The next
// item's weights are requested before the current one is worked on, the first one's before x is staged.  x lies in LDS
// as two planes, elements 8c .. 8c + 3 and 8c + 4 .. 8c + 7 of every chunk c, so that both 16-byte reads of a wave are
// free of bank conflicts.
// ---------------------------------------------------------------------------------------------------------------------
constexpr int GT = 512, GW = GT / 64; // threads and waves of a workgroup
struct GemvArgs {
    axq_parts parts;
    axq_in in;
    int steps; // of 512 elements
};

// Of a step of AXQ_IN_SEGMENTS: its weight's columns, their row pitch and 16-byte chunks; its inputs, their number and factor.
struct Step { const uint16_t *w; int ldw, c8; const float *x; float f; int k, glu; };

// Four inputs from e on, zeros past the end
__device__ inline f32x4 load_quad(const float *x, int e, int k) {
    if (e + 4 <= k) return *reinterpret_cast<const f32x4_any *>(x + e);
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < 4; i++)
        if (e + i < k) v[i] = x[e + i];
    return v;
}
__device__ inline f32x4 load_step(const Step &t, int e) {
    f32x4 v;
    if (t.glu) { // both halves are padded to whole groups
        const float *z = t.x + (e / AXQ_GLU_GROUP) * 2 * AXQ_GLU_GROUP + e % AXQ_GLU_GROUP;
        v = load_quad(z, 0, t.k - e) * load_quad(z + AXQ_GLU_GROUP, 0, t.k - e);
    } else {
        v = load_quad(t.x, e, t.k);
    }
    return v * t.f;
}

template <int MODE>
__device__ void stage_x(const GemvArgs &a, const axq_part &p, const Step *table, float *xs, float *scratch) {
    const axq_in &in = a.in;
    const float *mu = p.mu;
    const int k = in.k, tid = threadIdx.x, xl = a.steps * 512, half = xl >> 1, quads = xl >> 2;
    auto slot = [half](int e) { return ((e >> 3) << 2) + (e & 3) + ((e & 4) ? half : 0); };
    auto quad = [half, xs](int q) -> f32x4 & { return *reinterpret_cast<f32x4 *>(xs + ((q >> 1) << 2) + ((q & 1) ? half : 0)); };
    if (MODE == AXQ_IN_SEGMENTS) { // four loads under way per thread
        for (int q0 = tid; q0 < quads; q0 += 4 * GT) {
            f32x4 v[4];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int q = q0 + i * GT;
                if (q < quads) v[i] = load_step(table[q >> 7], (q & 127) << 2);
            }
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (q0 + i * GT < quads) quad(q0 + i * GT) = v[i];
        }
    } else if (MODE == AXQ_IN_LAYER_NORM) {
        constexpr int NW = 2; // the first quads' weights are requested with the inputs
        f32x4 w[NW];
        float sum = 0.f, ss = 0.f;
#pragma unroll
        for (int i = 0; i < NW; i++)
            if (tid + i * GT < quads) w[i] = load_quad(p.nw, (tid + i * GT) << 2, k);
        for (int q = tid; q < quads; q += GT) {
            const f32x4 v = load_quad(in.x, q << 2, k);
            quad(q) = v;
            sum += (v[0] + v[1]) + (v[2] + v[3]);
        }
        const float mean = axq_block_sum(sum, scratch) / (float)k;
        for (int q = tid; q < quads; q += GT) {
            const f32x4 v = quad(q);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float d = (q << 2) + i < k ? v[i] - mean : 0.f;
                ss = fmaf(d, d, ss);
            }
        }
        const float inv = 1.0f / sqrtf(axq_block_sum(ss, scratch) / (float)k + in.eps);
#pragma unroll
        for (int i = 0; i < NW; i++)
            if (tid + i * GT < quads) quad(tid + i * GT) = (quad(tid + i * GT) - mean) * inv * w[i]; // zeros past the end
        for (int q = tid + NW * GT; q < quads; q += GT) quad(q) = (quad(q) - mean) * inv * load_quad(p.nw, q << 2, k);
    } else
    if (MODE == AXQ_IN_RMS_GATE) {
        float ss = 0.f;
        for (int e = tid; e < k; e += GT) {
            const float v = in.x[e];
            xs[slot(e)] = v;
            ss = fmaf(v, v, ss);
        }
        ss = axq_block_sum(ss, scratch);
        const float inv = 1.0f / sqrtf(ss / (float)k + in.eps);
        for (int e = tid; e < xl; e += GT) xs[slot(e)] = e < k ? xs[slot(e)] * inv * in.nw[e] * in.gate[e] : 0.f;
    } else if (MODE == AXQ_IN_POLY_NORM) {
        float s1 = 0.f, s2 = 0.f, s3 = 0.f;
        for (int e = tid; e < k; e += GT) {
            const float z = in.x[e], z2 = z * z, z3 = z2 * z;
            xs[slot(e)] = z;
            s1 += z2; s2 = fmaf(z2, z2, s2); s3 = fmaf(z3, z3, s3);
        }
        s1 = axq_block_sum(s1, scratch);
        s2 = axq_block_sum(s2, scratch);
        s3 = axq_block_sum(s3, scratch);
        const float c1 = in.coef[0] / sqrtf(s1 / (float)k + in.eps), c2 = in.coef[1] / sqrtf(s2 / (float)k + in.eps);
        const float c3 = in.coef[2] / sqrtf(s3 / (float)k + in.eps), c0 = in.coef[3];
        for (int e = tid; e < xl; e += GT) {
            const float z = e < k ? xs[slot(e)] : 0.f;
            xs[slot(e)] = e < k ? fmaf(fmaf(fmaf(c3, z, c2), z, c1), z, c0) : 0.f;
        }
    } else {
        const float alpha = MODE == AXQ_IN_PLAIN ? 0.f : in.alpha[0];
        const bool first = MODE == AXQ_IN_TANH_NORM_MIX && in.pos[0] == 0;
        for (int e = tid; e < xl; e += GT) {
            float v = 0.f;
            if (e < k) {
                v = in.x[e];
                if (MODE != AXQ_IN_PLAIN) v = tanh_norm(v, alpha, in.nw[e], in.nb[e]);
                if (MODE == AXQ_IN_TANH_NORM_MIX && mu) {
                    const float p = first ? 0.f : in.prev[e];
                    v = fmaf(p - v, mu[e], v);
                }
            }
            xs[slot(e)] = v;
        }
    }
    __syncthreads();
}

template <int MODE, int R>
__global__ void __launch_bounds__(GT, 4) dense_gemv_kernel(GemvArgs a) {
    extern __shared__ __attribute__((aligned(16))) float xs[];
    __shared__ float scratch[16];
    constexpr bool SEG = MODE == AXQ_IN_SEGMENTS;
    __shared__ Step table[SEG ? AXQ_DENSE_MAX_K / 512 : 1];
    constexpr int U = 8 / R;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nb = a.parts.n_blocks, b0 = (int)((long long)nb * blockIdx.x / gridDim.x), b1 = (int)((long long)nb * (blockIdx.x + 1) / gridDim.x);
    const int half = a.steps * 256, k8 = (a.in.k + 7) >> 3;
    auto part_of_block = [&](int b) {
        int pi = 0;
        while (pi + 1 < a.parts.n_parts && b >= a.parts.p[pi + 1].blk0) pi++;
        return pi;
    };
    if (SEG) {
        for (int t = tid; t < a.steps; t += GT) {
            int si = 0;
            while (si + 1 < a.in.n_seg && t >= a.in.seg[si + 1].step0) si++;
            const axq_seg &g = a.in.seg[si];
            const int i = (t - g.step0) / g.steps, s = (t - g.step0) - i * g.steps;
            table[t].w = g.w + (size_t)(g.sel ? g.sel[i] : i) * g.stride + (size_t)s * 512;
            table[t].ldw = g.ldw;
            table[t].c8 = ((g.k + 7) >> 3) - s * 64;
            table[t].x = g.x + (size_t)i * g.ldx + (size_t)s * (g.glu ? 1024 : 512);
            table[t].f = g.scale ? g.scale[i] : 1.0f;
            table[t].k = g.k - s * 512;
            table[t].glu = g.glu;
        }
        __syncthreads();
    }
    // chunks past a row's end: a valid chunk against zeros; rows past the end: the last row, dropped
    auto request = [&](int b, int s0, u32x4 (&q)[U][R]) {
        const axq_part &p = a.parts.p[part_of_block(b)];
        const int row0 = ((b - p.blk0) * GW + wave) * R;
#pragma unroll
        for (int r = 0; r < R; r++) {
            int row = row0 + r < p.n ? row0 + r : p.n - 1;
            if (SEG) {
#pragma unroll
                for (int u = 0; u < U; u++) {
                    const Step &t = table[s0 + u < a.steps ? s0 + u : a.steps - 1];
                    const int c = lane < t.c8 ? lane : t.c8 - 1;
                    q[u][r] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(t.w + (size_t)row * t.ldw + (size_t)c * 8));
                }
                continue;
            }
            if (MODE == AXQ_IN_LAYER_NORM && p.sel) {
                const int i = row / p.sel_rows;
                row += (p.sel[i] - i) * p.sel_rows;
            }
            const uint16_t *w = p.w + (size_t)row * p.ldw;
#pragma unroll
            for (int u = 0; u < U; u++) {
                int c = (s0 + u) * 64 + lane;
                c = c < k8 ? c : k8 - 1;
                q[u][r] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(w + (size_t)c * 8));
            }
        }
    };
    u32x4 qa[U][R], qb[U][R];
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; r++) acc[r] = 0.f;
    int staged = -1;
    // one item: the products of block b from step s0 on, and at the row's end the results
    auto work = [&](int b, int s0, const u32x4 (&q)[U][R]) {
        const int pi = part_of_block(b);
        const axq_part &p = a.parts.p[pi];
        if (staged < 0 || (MODE == AXQ_IN_TANH_NORM_MIX && staged != pi) ||
            (MODE == AXQ_IN_LAYER_NORM && a.parts.p[staged].nw != p.nw)) { // the same for all waves
            if (staged >= 0) __syncthreads();
            stage_x<MODE>(a, p, table, xs, scratch);
            staged = pi;
        }
#pragma unroll
        for (int u = 0; u < U; u++) {
            if (s0 + u < a.steps) {
                const int c = (s0 + u) * 64 + lane;
                const float4 xa = *reinterpret_cast<const float4 *>(xs + c * 4), xb = *reinterpret_cast<const float4 *>(xs + half + c * 4);
#pragma unroll
                for (int r = 0; r < R; r++) {
                    float t = acc[r];
                    t = fmaf(axq_bf16_lo(q[u][r][0]), xa.x, t); t = fmaf(axq_bf16_hi(q[u][r][0]), xa.y, t);
                    t = fmaf(axq_bf16_lo(q[u][r][1]), xa.z, t); t = fmaf(axq_bf16_hi(q[u][r][1]), xa.w, t);
                    t = fmaf(axq_bf16_lo(q[u][r][2]), xb.x, t); t = fmaf(axq_bf16_hi(q[u][r][2]), xb.y, t);
                    t = fmaf(axq_bf16_lo(q[u][r][3]), xb.z, t); t = fmaf(axq_bf16_hi(q[u][r][3]), xb.w, t);
                    acc[r] = t;
                }
            }
        }
        if (s0 + U >= a.steps) {
#pragma unroll
            for (int r = 0; r < R; r++) acc[r] = axq_wave_sum(acc[r]);
            float v = acc[0];
#pragma unroll
            for (int r = 1; r < R; r++) v = lane == r ? acc[r] : v;
            const int row = ((b - p.blk0) * GW + wave) * R + lane;
            if (lane < R && row < p.n) {
                if (p.bias) v += p.bias[row];
                v = p.act == AXQ_ACT_GLU_GELU ? ((row & AXQ_GLU_GROUP) ? v : axq_gelu_tanh(v)) : axq_act(p.act, v, a.parts.cap);
                if (p.resid) v += p.resid[row];
                reinterpret_cast<float *>(p.y)[row] = v;
                if (p.avg.out) p.avg.out[row] = axq_average(p.avg, row, v);
            }
#pragma unroll
            for (int r = 0; r < R; r++) acc[r] = 0.f;
        }
    };
    auto advance = [&](int &b, int &s0) {
        s0 += U;
        if (s0 >= a.steps) { s0 = 0; b++; }
    };
    int b = b0, s0 = 0;
    if (b >= b1) return;
    request(b, s0, qa);
    while (true) {
        int nb1 = b, ns1 = s0;
        advance(nb1, ns1);
        if (nb1 < b1) request(nb1, ns1, qb);
        work(b, s0, qa);
        if (nb1 >= b1) break;
        b = nb1; s0 = ns1;
        advance(b, s0);
        if (b < b1) request(b, s0, qa);
        work(nb1, ns1, qb);
        if (b >= b1) break;
    }
}

template <int MODE, int R>
int launch_gemv(axq_ctx *ctx, GemvArgs &a) {
    int nb = 0;
    for (int i = 0; i < a.parts.n_parts; i++) {
        a.parts.p[i].blk0 = nb;
        nb += (a.parts.p[i].n + GW * R - 1) / (GW * R);
    }
    a.parts.n_blocks = nb;
    const size_t lds = (size_t)a.steps * 512 * sizeof(float);
    const int most = (lds > 76 * 1024 ? 1 : 2) * ctx->prop.multiProcessorCount; // as many as are there at once
    static std::atomic<uint64_t> lds_allowed{0};
    int rc;
    if (lds > 48 * 1024 &&
        (rc = axq_allow_lds(ctx, reinterpret_cast<const void *>(&dense_gemv_kernel<MODE, R>), lds_allowed, (size_t)AXQ_DENSE_MAX_K * 4)))
        return rc;
    dense_gemv_kernel<MODE, R><<<nb < most ? nb : most, GT, lds, ctx->stream>>>(a);
    AXQ_LAUNCH_CHECK(ctx, "dense_gemv_kernel");
    return AXQ_OK;
}

template <int MODE>
int launch_gemv_mode(axq_ctx *ctx, GemvArgs &a) {
    long long rows = 0;
    for (int i = 0; i < a.parts.n_parts; i++) rows += a.parts.p[i].n;
    if (rows >= 8192) return launch_gemv<MODE, 2>(ctx, a);
    return launch_gemv<MODE, 1>(ctx, a);
}

// ---------------------------------------------------------------------------------------------------------------------
// GEMM on bf16 rows: tiles of BM x BN, K in steps of 64, operands straight from memory into LDS (16 bytes per lane,
// two stages).  Row r of a tile is 128 bytes of LDS whose 16-byte pieces are exchanged by r & 7 (the loads take the
// permuted source address, the destination being fixed), so that the operand reads of eight rows use all banks.
// The product is taken as D[row of x][row of W]: a lane's accumulators are one output column.
// ---------------------------------------------------------------------------------------------------------------------
struct GemmArgs {
    axq_parts parts;
    int m, k, ldx, mt, tiles;
    axq_groups g; // grouped form
};

// A product's result on its way out (act_done: the activation has been applied)
__device__ inline void finish(const axq_part &p, float cap, int m, int n, float v, bool act_done = false) {
    if (p.bias) v += p.bias[n];
    if (!act_done) v = axq_act(p.act, v, cap);
    if (p.scale) v *= p.scale[m];
    const size_t i = (size_t)m * p.ldy + n;
    if (p.resid) v += p.resid[i];
    if (p.out16) reinterpret_cast<uint16_t *>(p.y)[i] = axq_to_bf16(v);
    else reinterpret_cast<float *>(p.y)[i] = v;
}

// ... and, once a thread's results are written, the mean over the layers at one of them
__device__ inline void finish_mean(const axq_part &p, int m, int n) {
    const size_t i = (size_t)m * p.ldy + n;
    p.avg.out[i] = axq_average(p.avg, i, reinterpret_cast<const float *>(p.y)[i]);
}

// Which rows and which weight a workgroup of a grouped product has: row tile `t` -> false if there is no such tile.
__device__ inline bool group_tile(const axq_groups &g, int t, int &m0, int &m1, size_t &woff) {
    if (t >= g.tiles[0]) return false;
    const int32_t *e = g.tiles + 4 + 4 * t;
    woff = (size_t)e[0] * g.stride;
    m0 = e[1];
    m1 = e[2];
    return true;
}

__device__ inline int acc_row(int r, int lane) { return 8 * (r >> 2) + 4 * (lane >> 5) + (r & 3); }

// Tiles in an order that gives each XCD (workgroups go round them) a contiguous run; a run walks the row tiles of a
// column tile first, so that a weight tile is read by one XCD's L2.
__device__ inline int xcd_tile(int tiles) {
    const int b = blockIdx.x, per = tiles >> 3, rest = tiles & 7, x = b & 7;
    return x * per + (x < rest ? x : rest) + (b >> 3);
}

template <int BM, int BN, bool GROUPED>
__global__ void __launch_bounds__(256) dense_gemm_kernel(GemmArgs a) {
    constexpr int MT = BM / 64, NT = BN / 64;          // 32 x 32 tiles of a wave (2 x 2 waves)
    constexpr int AL = BM / 32, BL = BN / 32;          // 16-byte loads per thread and step
    __shared__ __attribute__((aligned(16))) uint16_t lds[2][(BM + BN) * 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave >> 1, wn = wave & 1;
    const int tile = xcd_tile(a.tiles), ct = tile / a.mt;
    int m0 = (tile - ct * a.mt) * BM, m1 = a.m, pi = 0;
    size_t woff = 0;
    if (GROUPED && !group_tile(a.g, tile - ct * a.mt, m0, m1, woff)) return;
    while (!GROUPED && pi + 1 < a.parts.n_parts && ct >= a.parts.p[pi + 1].blk0) pi++;
    const axq_part &p = a.parts.p[pi];
    const int n0 = (ct - p.blk0) * BN;
    const uint16_t *x = reinterpret_cast<const uint16_t *>(p.x);

    const uint16_t *ga[AL], *gb[BL];
#pragma unroll
    for (int i = 0; i < AL; i++) {
        const int idx = (i * 4 + wave) * 64 + lane, r = idx >> 3, c = (idx & 7) ^ (r & 7);
        int row = m0 + r < m1 ? m0 + r : m1 - 1;
        if (GROUPED && a.g.src) row = a.g.src[row];
        ga[i] = x + (size_t)row * a.ldx + c * 8;
    }
#pragma unroll
    for (int i = 0; i < BL; i++) {
        const int idx = (i * 4 + wave) * 64 + lane, r = idx >> 3, c = (idx & 7) ^ (r & 7);
        const int row = n0 + r < p.n ? n0 + r : p.n - 1;
        gb[i] = p.w + woff + (size_t)row * p.ldw + c * 8;
    }
    auto fetch = [&](int stage, int kt) {
        uint16_t *la = lds[stage], *lb = la + BM * 64;
#pragma unroll
        for (int i = 0; i < AL; i++)
            __builtin_amdgcn_global_load_lds((gbl_void *)(ga[i] + kt * 64), (lds_void *)(la + (i * 4 + wave) * 512), 16, 0, 0);
#pragma unroll
        for (int i = 0; i < BL; i++)
            __builtin_amdgcn_global_load_lds((gbl_void *)(gb[i] + kt * 64), (lds_void *)(lb + (i * 4 + wave) * 512), 16, 0, 0);
    };
    f32x16 acc[MT][NT];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < NT; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) acc[i][j][r] = 0.f;

    const int kts = a.k >> 6, li = lane & 31, lh = lane >> 5;
    fetch(0, 0);
    for (int kt = 0; kt < kts; kt++) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); // this step's tile is in LDS ...
        __syncthreads();                                  // ... of every wave, and nobody reads the other stage any more
        if (kt + 1 < kts) fetch((kt + 1) & 1, kt + 1);
        const uint16_t *la = lds[kt & 1], *lb = la + BM * 64;
#pragma unroll
        for (int ks = 0; ks < 4; ks++) {
            bf16x8 fa[MT], fb[NT];
#pragma unroll
            for (int i = 0; i < MT; i++) {
                const int r = wm * (BM / 2) + i * 32 + li;
                fa[i] = *reinterpret_cast<const bf16x8 *>(la + r * 64 + (((ks * 2 + lh) ^ (r & 7)) << 3));
            }
#pragma unroll
            for (int j = 0; j < NT; j++) {
                const int r = wn * (BN / 2) + j * 32 + li;
                fb[j] = *reinterpret_cast<const bf16x8 *>(lb + r * 64 + (((ks * 2 + lh) ^ (r & 7)) << 3));
            }
#pragma unroll
            for (int i = 0; i < MT; i++)
#pragma unroll
                for (int j = 0; j < NT; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
        }
    }
    if (NT == 2 && p.act == AXQ_ACT_GLU_GELU) { // a wave's two column tiles are a group of gates and its ups
        const int n = n0 / 2 + wn * 32 + li;
        if (n >= p.n / 2) return;
#pragma unroll
        for (int i = 0; i < MT; i++)
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int m = m0 + wm * (BM / 2) + i * 32 + acc_row(r, lane);
                if (m < m1) finish(p, a.parts.cap, m, n, axq_gelu_tanh(acc[i][0][r]) * acc[i][NT - 1][r], true);
            }
        return;
    }
#pragma unroll
    for (int j = 0; j < NT; j++) {
        const int n = n0 + wn * (BN / 2) + j * 32 + li;
        if (n >= p.n) continue;
#pragma unroll
        for (int i = 0; i < MT; i++)
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int m = m0 + wm * (BM / 2) + i * 32 + acc_row(r, lane);
                if (m < m1) finish(p, a.parts.cap, m, n, acc[i][j][r]);
            }
    }
    if (!GROUPED && p.avg.out) {
#pragma clang loop unroll(disable)
        for (int x = 0; x < NT * MT * 16; x++) {
            const int n = n0 + wn * (BN / 2) + (x & (NT - 1)) * 32 + li, m = m0 + wm * (BM / 2) + x / (NT * 16) * 32 + acc_row((x / NT) & 15, lane);
            if (n < p.n && m < m1) finish_mean(p, m, n);
        }
    }
}

// GEMM on f32 rows in true 32-bit: 64 x 64 tiles, 4 x 4 results per thread, K in steps of 16.
template <bool GROUPED>
__global__ void __launch_bounds__(256) dense_gemm_f32_kernel(GemmArgs a) {
    __shared__ __attribute__((aligned(16))) float as[16][68], bs[16][68];
    const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
    const int tile = xcd_tile(a.tiles), ct = tile / a.mt;
    int m0 = (tile - ct * a.mt) * 64, m1 = a.m, pi = 0;
    size_t woff = 0;
    if (GROUPED && !group_tile(a.g, tile - ct * a.mt, m0, m1, woff)) return;
    while (!GROUPED && pi + 1 < a.parts.n_parts && ct >= a.parts.p[pi + 1].blk0) pi++;
    const axq_part &p = a.parts.p[pi];
    const int n0 = (ct - p.blk0) * 64;
    const float *x = reinterpret_cast<const float *>(p.x);
    const int lr = tid >> 2, lc = (tid & 3) * 4; // this thread's four elements of a step: row lr, columns lc ..
    int row = m0 + lr < m1 ? m0 + lr : m1 - 1;
    if (GROUPED && a.g.src) row = a.g.src[row];
    const float *ga = x + (size_t)row * a.ldx + lc;
    const uint16_t *gb = p.w + woff + (size_t)(n0 + lr < p.n ? n0 + lr : p.n - 1) * p.ldw + lc;
    float acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) acc[i][j] = 0.f;
    for (int k = 0; k < a.k; k += 16) {
        const float4 va = *reinterpret_cast<const float4 *>(ga + k);
        const uint2 vb = *reinterpret_cast<const uint2 *>(gb + k);
        __syncthreads();
        as[lc][lr] = va.x; as[lc + 1][lr] = va.y; as[lc + 2][lr] = va.z; as[lc + 3][lr] = va.w;
        bs[lc][lr] = axq_bf16_lo(vb.x); bs[lc + 1][lr] = axq_bf16_hi(vb.x); bs[lc + 2][lr] = axq_bf16_lo(vb.y); bs[lc + 3][lr] = axq_bf16_hi(vb.y);
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < 16; kk++) {
            const float4 fa = *reinterpret_cast<const float4 *>(&as[kk][ty * 4]), fb = *reinterpret_cast<const float4 *>(&bs[kk][tx * 4]);
            const float av[4] = {fa.x, fa.y, fa.z, fa.w}, bv[4] = {fb.x, fb.y, fb.z, fb.w};
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i][j] = fmaf(av[i], bv[j], acc[i][j]);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int m = m0 + ty * 4 + i, n = n0 + tx * 4 + j;
            if (m < m1 && n < p.n) {
                const bool glu = p.act == AXQ_ACT_GLU_GELU;
                finish(p, a.parts.cap, m, n, glu && !(n & AXQ_GLU_GROUP) ? axq_gelu_tanh(acc[i][j]) : acc[i][j], glu);
                if (!GROUPED && p.avg.out) finish_mean(p, m, n);
            }
        }
}

int count_tiles(GemmArgs &a, int bm, int bn) {
    int ct = 0;
    for (int i = 0; i < a.parts.n_parts; i++) {
        a.parts.p[i].blk0 = ct;
        ct += (a.parts.p[i].n + bn - 1) / bn;
    }
    a.parts.n_blocks = ct;
    a.mt = (a.m + bm - 1) / bm;
    return a.tiles = ct * a.mt;
}

// ---------------------------------------------------------------------------------------------------------------------
// Row operations of a prompt, one workgroup per row.
// ---------------------------------------------------------------------------------------------------------------------
__device__ inline void put(const axq_rows_out &o, size_t row, int e, float v) {
    if (o.f32) reinterpret_cast<float *>(o.x)[row * o.ldx + e] = v;
    else reinterpret_cast<uint16_t *>(o.x)[row * o.ldx + e] = axq_to_bf16(v);
}

__device__ inline void put_quad(const axq_rows_out &o, size_t row, int e, f32x4 v) { // e and rows: multiples of 4
    if (o.f32) *reinterpret_cast<f32x4 *>(reinterpret_cast<float *>(o.x) + row * o.ldx + e) = v;
    else
        *reinterpret_cast<uint2 *>(reinterpret_cast<uint16_t *>(o.x) + row * o.ldx + e) =
            make_uint2(axq_to_bf16(v[0]) | (uint32_t)axq_to_bf16(v[1]) << 16, axq_to_bf16(v[2]) | (uint32_t)axq_to_bf16(v[3]) << 16);
}

__global__ void __launch_bounds__(256) embed_pos_kernel(const uint16_t *emb16, const float *emb32, const float *pos_table, const int32_t *tok,
                                                        const int32_t *pos, int pos0, int width, float *h) {
    const int e = blockIdx.x * 256 + threadIdx.x, t = blockIdx.y;
    if (e >= width) return;
    const int p = pos ? pos[0] + t : pos0 + t;
    const size_t i = (size_t)tok[t] * width + e;
    const float v = emb32 ? emb32[i] : (float)__builtin_bit_cast(_Float16, emb16[i]);
    h[(size_t)t * width + e] = pos_table ? v + pos_table[(size_t)p * width + e] : v;
}

struct MixPtrs { const float *mu[AXQ_MAX_PARTS]; };

__global__ void __launch_bounds__(256) rows_tanh_norm_kernel(axq_in in, int m, int first, int n_mix, MixPtrs mix, axq_rows_out out) {
    const int t = blockIdx.x;
    const float alpha = in.alpha[0];
    const float *h = in.x + (size_t)(in.rows ? in.rows[t] : t) * in.k;
    for (int e = threadIdx.x; e < out.ldx; e += 256) {
        const bool in_row = e < in.k;
        const float nw = in_row ? in.nw[e] : 0.f, nb = in_row ? in.nb[e] : 0.f;
        const float n = in_row ? tanh_norm(h[e], alpha, nw, nb) : 0.f;
        if (n_mix == 0) {
            put(out, t, e, n);
            continue;
        }
        float p = 0.f;
        if (in_row && t > 0) p = tanh_norm(h[e - in.k], alpha, nw, nb);
        else if (in_row && !first) p = in.prev[e];
        for (int i = 0; i < n_mix; i++) put(out, (size_t)i * m + t, e, in_row ? fmaf(p - n, mix.mu[i][e], n) : 0.f);
    }
}

__global__ void __launch_bounds__(256) store_prev_kernel(axq_in in, int m, float *prev) {
    const int e = blockIdx.x * 256 + threadIdx.x;
    if (e < in.k) prev[e] = tanh_norm(in.x[(size_t)(m - 1) * in.k + e], in.alpha[0], in.nw[e], in.nb[e]);
}

// one workgroup per row and group (the last group's workgroup zeroes the tail)
__global__ void __launch_bounds__(256) rows_rms_gate_kernel(axq_in in, int group, axq_rows_out out) {
    __shared__ float scratch[16];
    const int t = blockIdx.x, e0 = blockIdx.y * group;
    const float *x = in.x + (size_t)t * in.k, *g = in.gate + (size_t)t * in.k;
    float ss = 0.f;
    for (int e = e0 + threadIdx.x; e < e0 + group; e += blockDim.x) ss = fmaf(x[e], x[e], ss);
    ss = axq_block_sum(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)group + in.eps);
    for (int e = e0 + threadIdx.x; e < e0 + group; e += blockDim.x) put(out, t, e, x[e] * inv * in.nw[e] * g[e]);
    if (blockIdx.y == gridDim.y - 1)
        for (int e = in.k + threadIdx.x; e < out.ldx; e += blockDim.x) put(out, t, e, 0.f);
}

__global__ void __launch_bounds__(256) rows_poly_norm_kernel(axq_in in, axq_rows_out out) {
    __shared__ float scratch[16];
    const int t = blockIdx.x, k = in.k;
    const float *x = in.x + (size_t)t * k;
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
    for (int e = threadIdx.x; e < k; e += 256) {
        const float z = x[e], z2 = z * z, z3 = z2 * z;
        s1 += z2; s2 = fmaf(z2, z2, s2); s3 = fmaf(z3, z3, s3);
    }
    s1 = axq_block_sum(s1, scratch);
    s2 = axq_block_sum(s2, scratch);
    s3 = axq_block_sum(s3, scratch);
    const float c1 = in.coef[0] / sqrtf(s1 / (float)k + in.eps), c2 = in.coef[1] / sqrtf(s2 / (float)k + in.eps);
    const float c3 = in.coef[2] / sqrtf(s3 / (float)k + in.eps), c0 = in.coef[3];
    for (int e = threadIdx.x; e < out.ldx; e += 256) {
        const float z = e < k ? x[e] : 0.f;
        put(out, t, e, e < k ? fmaf(fmaf(fmaf(c3, z, c2), z, c1), z, c0) : 0.f);
    }
}

__global__ void __launch_bounds__(256) rows_layer_norm_kernel(axq_in in, const float *nw1, axq_rows_out out1, const float *nw2, axq_rows_out out2) {
    __shared__ float scratch[16];
    constexpr int NR = 4; // quads of a row that a thread keeps; wider rows are read again
    const int t = blockIdx.x, k = in.k, tid = threadIdx.x, quads = out1.ldx >> 2;
    const float *x = in.x + (size_t)(in.rows ? in.rows[t] : t) * k;
    f32x4 r[NR];
    float sum = 0.f, ss = 0.f;
#pragma unroll
    for (int i = 0; i < NR; i++) {
        r[i] = tid + i * 256 < quads ? load_quad(x, (tid + i * 256) << 2, k) : f32x4{0.f, 0.f, 0.f, 0.f};
        sum += (r[i][0] + r[i][1]) + (r[i][2] + r[i][3]);
    }
    for (int e = NR * 1024 + tid; e < k; e += 256) sum += x[e];
    const float mean = axq_block_sum(sum, scratch) / (float)k;
#pragma unroll
    for (int i = 0; i < NR; i++)
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const float d = ((tid + i * 256) << 2) + c < k ? r[i][c] - mean : 0.f;
            ss = fmaf(d, d, ss);
        }
    for (int e = NR * 1024 + tid; e < k; e += 256) {
        const float d = x[e] - mean;
        ss = fmaf(d, d, ss);
    }
    const float inv = 1.0f / sqrtf(axq_block_sum(ss, scratch) / (float)k + in.eps);
#pragma unroll
    for (int i = 0; i < NR; i++) {
        const int q = tid + i * 256;
        if (q >= quads) break;
        const f32x4 n = (r[i] - mean) * inv; // past the end the weights are zeros
        put_quad(out1, t, q << 2, n * load_quad(nw1, q << 2, k));
        if (nw2) put_quad(out2, t, q << 2, n * load_quad(nw2, q << 2, k));
    }
    for (int e = NR * 1024 + tid; e < out1.ldx; e += 256) {
        const float n = e < k ? (x[e] - mean) * inv : 0.f;
        put(out1, t, e, e < k ? n * nw1[e] : 0.f);
        if (nw2) put(out2, t, e, e < k ? n * nw2[e] : 0.f);
    }
}

__global__ void __launch_bounds__(256) rows_glu_kernel(const float *z, int ldz, int k, axq_rows_out out) {
    const float *row = z + (size_t)blockIdx.x * ldz;
    for (int e = threadIdx.x; e < out.ldx; e += 256) {
        const float *g = row + (e / AXQ_GLU_GROUP) * 2 * AXQ_GLU_GROUP + e % AXQ_GLU_GROUP;
        put(out, blockIdx.x, e, e < k ? g[0] * g[AXQ_GLU_GROUP] : 0.f);
    }
}

__global__ void __launch_bounds__(64) rows_zero_tail_kernel(int k, axq_rows_out out) {
    for (int e = k + threadIdx.x; e < out.ldx; e += 64) put(out, blockIdx.x, e, 0.f);
}

} // namespace

int axq_dense_gemv(axq_ctx *ctx, int mode, const axq_in &in, axq_parts &parts) {
    if ((mode != AXQ_IN_SEGMENTS && (in.k < 1 || in.k > AXQ_DENSE_MAX_K)) || parts.n_parts < 1 || parts.n_parts > AXQ_MAX_PARTS)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: a decode product takes 1 to %d inputs and 1 to %d weights, got %d and %d",
                        AXQ_DENSE_MAX_K, AXQ_MAX_PARTS, in.k, parts.n_parts);
    GemvArgs a;
    a.parts = parts;
    a.in = in;
    a.steps = (in.k + 511) / 512;
    if (mode == AXQ_IN_SEGMENTS) {
        a.steps = 0;
        int items = 0;
        for (int i = 0; i < in.n_seg; i++) {
            axq_seg &g = a.in.seg[i];
            if (g.k < 1 || g.count < 1) return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: segment %d of %d x %d elements", i, g.count, g.k);
            g.step0 = a.steps;
            g.steps = (g.k + 511) / 512;
            a.steps += g.count * g.steps;
            items += g.count;
        }
        if (in.n_seg < 1 || in.n_seg > AXQ_MAX_SEGS || items > AXQ_MAX_SEG_ITEMS || a.steps > AXQ_DENSE_MAX_K / 512 || parts.n_parts != 1)
            return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: a decode product over %d steps of 512 (at most %d)", a.steps, AXQ_DENSE_MAX_K / 512);
    }
    switch (mode) {
    case AXQ_IN_PLAIN: return launch_gemv_mode<AXQ_IN_PLAIN>(ctx, a);
    case AXQ_IN_TANH_NORM: return launch_gemv_mode<AXQ_IN_TANH_NORM>(ctx, a);
    case AXQ_IN_TANH_NORM_MIX: return launch_gemv_mode<AXQ_IN_TANH_NORM_MIX>(ctx, a);
    case AXQ_IN_RMS_GATE: return launch_gemv_mode<AXQ_IN_RMS_GATE>(ctx, a);
    case AXQ_IN_POLY_NORM: return launch_gemv_mode<AXQ_IN_POLY_NORM>(ctx, a);
    case AXQ_IN_LAYER_NORM: return launch_gemv_mode<AXQ_IN_LAYER_NORM>(ctx, a);
    case AXQ_IN_SEGMENTS: return launch_gemv_mode<AXQ_IN_SEGMENTS>(ctx, a);
    default: return axq_fail(ctx, AXQ_ERR_INVALID_ARGUMENT, "axq_dense_gemv: unknown input mode %d", mode);
    }
}

int axq_dev_dense_gemv(axq_ctx *ctx, const axq_weight *w, const float *x, const float *bias, float *y) {
    axq_in in;
    in.x = x;
    in.k = (int)w->k;
    axq_parts parts = {};
    parts.n_parts = 1;
    parts.p[0].w = reinterpret_cast<const uint16_t *>(w->codes);
    parts.p[0].ldw = (int)(w->codes_pitch / 2);
    parts.p[0].n = (int)w->n_rows;
    parts.p[0].bias = bias;
    parts.p[0].y = y;
    return axq_dense_gemv(ctx, AXQ_IN_PLAIN, in, parts);
}

int axq_dense_gemm(axq_ctx *ctx, axq_parts &parts, int m, int k, int ldx, bool f32) {
    GemmArgs a;
    a.parts = parts;
    a.m = m;
    a.k = (k + 63) / 64 * 64;
    a.ldx = ldx;
    if (m < 1 || k < 1 || ldx % 64 != 0 || ldx < a.k || parts.n_parts < 1 || parts.n_parts > AXQ_MAX_PARTS)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: %d rows of %d elements (%d apart), %d weights", m, k, ldx, parts.n_parts);
    for (int i = 0; i < parts.n_parts; i++)
        if (parts.p[i].ldw < a.k || parts.p[i].n < 1)
            return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: weight %d has rows of %d elements, %d wanted", i, parts.p[i].ldw, a.k);
    bool glu = false;
    for (int i = 0; i < parts.n_parts; i++) glu |= parts.p[i].act == AXQ_ACT_GLU_GELU;
    if (f32) {
        count_tiles(a, 64, 64);
        dense_gemm_f32_kernel<false><<<a.tiles, 256, 0, ctx->stream>>>(a);
    } else if (m > 64 && count_tiles(a, 128, 128) >= ctx->prop.multiProcessorCount) {
        dense_gemm_kernel<128, 128, false><<<a.tiles, 256, 0, ctx->stream>>>(a);
    } else if (glu) {
        count_tiles(a, 64, 128);
        dense_gemm_kernel<64, 128, false><<<a.tiles, 256, 0, ctx->stream>>>(a);
    } else {
        count_tiles(a, 64, 64);
        dense_gemm_kernel<64, 64, false><<<a.tiles, 256, 0, ctx->stream>>>(a);
    }
    AXQ_LAUNCH_CHECK(ctx, "dense_gemm_kernel");
    return AXQ_OK;
}

int axq_dense_gemm_rows_per_tile(int rows, int groups, bool f32) { return !f32 && rows >= 96 * groups ? 128 : 64; }

int axq_dense_gemm_grouped(axq_ctx *ctx, axq_part &part, const axq_groups &g, int k, int ldx, bool f32) {
    GemmArgs a;
    a.parts = {};
    a.parts.p[0] = part;
    a.parts.n_parts = 1;
    a.m = 0;
    a.k = (k + 63) / 64 * 64;
    a.ldx = ldx;
    a.g = g;
    if (k < 1 || ldx % 64 != 0 || ldx < a.k || part.ldw < a.k || part.n < 1 || g.max_tiles < 1 || (g.bm != 64 && g.bm != 128))
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: grouped rows of %d elements (%d apart) against rows of %d", k, ldx, part.ldw);
    const int bn = f32 ? 64 : (g.bm == 128 ? 128 : 64);
    a.mt = g.max_tiles;
    a.tiles = (part.n + bn - 1) / bn * a.mt;
    if (f32) dense_gemm_f32_kernel<true><<<a.tiles, 256, 0, ctx->stream>>>(a);
    else if (g.bm == 128) dense_gemm_kernel<128, 128, true><<<a.tiles, 256, 0, ctx->stream>>>(a);
    else dense_gemm_kernel<64, 64, true><<<a.tiles, 256, 0, ctx->stream>>>(a);
    AXQ_LAUNCH_CHECK(ctx, "grouped dense_gemm_kernel");
    return AXQ_OK;
}

int axq_rows_embed(axq_ctx *ctx, const uint16_t *emb16, const float *emb32, const float *pos_table, const int32_t *tok, const int32_t *pos,
                   int pos0, int m, int width, float *h) {
    embed_pos_kernel<<<dim3((width + 255) / 256, m), 256, 0, ctx->stream>>>(emb16, emb32, pos_table, tok, pos, pos0, width, h);
    AXQ_LAUNCH_CHECK(ctx, "embed_pos_kernel");
    return AXQ_OK;
}

int axq_rows_tanh_norm(axq_ctx *ctx, const axq_in &in, int m, bool first, int n_mix, const float *const *mu, axq_rows_out out) {
    MixPtrs mix = {};
    for (int i = 0; i < n_mix; i++) mix.mu[i] = mu[i];
    rows_tanh_norm_kernel<<<m, 256, 0, ctx->stream>>>(in, m, first ? 1 : 0, n_mix, mix, out);
    AXQ_LAUNCH_CHECK(ctx, "rows_tanh_norm_kernel");
    return AXQ_OK;
}

int axq_store_prev(axq_ctx *ctx, const axq_in &in, int m, float *prev) {
    store_prev_kernel<<<(in.k + 255) / 256, 256, 0, ctx->stream>>>(in, m, prev);
    AXQ_LAUNCH_CHECK(ctx, "store_prev_kernel");
    return AXQ_OK;
}

int axq_rows_rms_gate(axq_ctx *ctx, const axq_in &in, int m, int group, axq_rows_out out) {
    rows_rms_gate_kernel<<<dim3(m, in.k / group), group <= 128 ? 64 : 256, 0, ctx->stream>>>(in, group, out);
    AXQ_LAUNCH_CHECK(ctx, "rows_rms_gate_kernel");
    return AXQ_OK;
}

int axq_rows_poly_norm(axq_ctx *ctx, const axq_in &in, int m, axq_rows_out out) {
    rows_poly_norm_kernel<<<m, 256, 0, ctx->stream>>>(in, out);
    AXQ_LAUNCH_CHECK(ctx, "rows_poly_norm_kernel");
    return AXQ_OK;
}

int axq_rows_layer_norm(axq_ctx *ctx, const axq_in &in, int m, const float *nw1, axq_rows_out out1, const float *nw2, axq_rows_out out2) {
    if (out1.ldx % 4) return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: layer norms of rows %d apart", out1.ldx);
    if (nw2 && out2.ldx != out1.ldx) return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: layer norms of rows %d and %d apart", out1.ldx, out2.ldx);
    rows_layer_norm_kernel<<<m, 256, 0, ctx->stream>>>(in, nw1, out1, nw2, out2);
    AXQ_LAUNCH_CHECK(ctx, "rows_layer_norm_kernel");
    return AXQ_OK;
}

int axq_rows_glu(axq_ctx *ctx, const float *z, int ldz, int k, int m, axq_rows_out out) {
    rows_glu_kernel<<<m, 256, 0, ctx->stream>>>(z, ldz, k, out);
    AXQ_LAUNCH_CHECK(ctx, "rows_glu_kernel");
    return AXQ_OK;
}

int axq_rows_zero_tail(axq_ctx *ctx, int m, int k, axq_rows_out out) {
    if (k == out.ldx) return AXQ_OK;
    rows_zero_tail_kernel<<<m, 64, 0, ctx->stream>>>(k, out);
    AXQ_LAUNCH_CHECK(ctx, "rows_zero_tail_kernel");
    return AXQ_OK;
}
