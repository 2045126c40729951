// Mixtures of experts: which experts a token goes through, its rows sorted by expert for the grouped products, and the
// weighted sum of what they gave.  Scores, choices and weights are f32.
#include "axq_dense.h"

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

// Best of the wave's candidates (value, index; index < 0: none), ties to the lower index.
__device__ inline int wave_argmax(float v, int i) {
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
        const float ov = __shfl_xor(v, d);
        const int oi = __shfl_xor(i, d);
        if (oi >= 0 && (i < 0 || ov > v || (ov == v && oi < i))) { v = ov; i = oi; }
    }
    return __builtin_amdgcn_readfirstlane(i);
}

__device__ inline float lane_of(float v, int lane) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), lane)); }

// Up to 64 experts: a wave per row, a lane per expert.  Places are counted: how many of the others come before this one.
__global__ void __launch_bounds__(64) route_lanes_kernel(axq_moe_router r, const float *z, int ldz, int32_t *sel, float *wt) {
    const int t = blockIdx.x, e = threadIdx.x, per = r.experts / r.groups, group = e / per;
    float s = e < r.experts ? axq_sigmoid(z[(size_t)t * ldz + e]) : 0.f;
    if (!(s == s)) s = 0.f; // with NaN among them places would not be distinct, and `sel` must hold experts whatever comes
    bool usable = e < r.experts;
    if (r.keep < r.groups) {
        float a = 0.f, b = 0.f; // scores are positive; a group of one has no second
        for (int j = 0; j < r.experts; j++) {
            const float v = lane_of(s, j);
            if (j / per == group) {
                b = fmaxf(b, fminf(a, v));
                a = fmaxf(a, v);
            }
        }
        const float mine = a + b;
        int before = 0;
        for (int g = 0; g < r.groups; g++) {
            const float v = lane_of(mine, g * per);
            before += v > mine || (v == mine && g < group);
        }
        usable = usable && before < r.keep;
    }
    const uint64_t others = __builtin_amdgcn_ballot_w64(usable);
    int before = 0;
    for (int j = 0; j < r.experts; j++) {
        const float v = lane_of(s, j);
        before += ((others >> j) & 1) && (v > s || (v == s && j < e));
    }
    const bool chosen = usable && before < r.top;
    const float inv = 1.0f / (axq_wave_sum(chosen ? s : 0.f) + 1e-20f);
    if (chosen) {
        sel[(size_t)t * r.top + before] = e;
        wt[(size_t)t * r.top + before] = s * inv;
    }
}

// Any number of experts: one wave per row.
__global__ void __launch_bounds__(64) route_kernel(axq_moe_router r, const float *z, int ldz, int32_t *sel, float *wt) {
    __shared__ float score[AXQ_MOE_MAX_EXPERTS], group[AXQ_MOE_MAX_EXPERTS];
    __shared__ int chosen[AXQ_MOE_MAX_EXPERTS];
    __shared__ uint8_t usable[AXQ_MOE_MAX_EXPERTS], kept[AXQ_MOE_MAX_EXPERTS];
    const int t = blockIdx.x, lane = threadIdx.x, per = r.experts / r.groups;
    for (int e = lane; e < r.experts; e += 64) {
        score[e] = axq_sigmoid(z[(size_t)t * ldz + e]);
        usable[e] = r.keep >= r.groups;
    }
    __syncthreads();
    if (r.keep < r.groups) {
        for (int g = lane; g < r.groups; g += 64) {
            float a = 0.f, b = 0.f; // scores are positive; a group of one has no second
            for (int e = g * per; e < (g + 1) * per; e++) {
                const float s = score[e];
                if (s > a) { b = a; a = s; }
                else if (s > b) b = s;
            }
            group[g] = a + b;
            kept[g] = 0;
        }
        __syncthreads();
        for (int n = 0; n < r.keep; n++) {
            float v = 0.f;
            int i = -1;
            for (int g = lane; g < r.groups; g += 64)
                if (!kept[g] && (i < 0 || group[g] > v)) { v = group[g]; i = g; }
            i = wave_argmax(v, i);
            __syncthreads();
            if (lane == 0) kept[i] = 1;
            for (int e = lane; e < per; e += 64) usable[i * per + e] = 1;
            __syncthreads();
        }
    }
    float sum = 0.f;
    for (int n = 0; n < r.top; n++) {
        float v = 0.f;
        int i = -1;
        for (int e = lane; e < r.experts; e += 64)
            if (usable[e] && (i < 0 || score[e] > v)) { v = score[e]; i = e; }
        i = wave_argmax(v, i);
        __syncthreads();
        if (lane == 0) {
            usable[i] = 0;
            chosen[n] = i;
        }
        sum += score[i];
        __syncthreads();
    }
    const float inv = 1.0f / (sum + 1e-20f);
    for (int n = lane; n < r.top; n += 64) {
        sel[(size_t)t * r.top + n] = chosen[n];
        wt[(size_t)t * r.top + n] = score[chosen[n]] * inv;
    }
}

// One workgroup (a thread per expert): entries counted per expert, slots handed out, row tiles listed.
__global__ void __launch_bounds__(1024) sort_kernel(const int32_t *sel, int n, int top, int experts, int bm, int32_t *slot_of, int32_t *src, int32_t *tiles) {
    __shared__ int count[AXQ_MOE_MAX_EXPERTS], start[AXQ_MOE_MAX_EXPERTS], tile0[AXQ_MOE_MAX_EXPERTS];
    const int tid = threadIdx.x;
    count[tid] = 0;
    __syncthreads();
    for (int i = tid; i < n; i += 1024) atomicAdd(&count[sel[i]], 1);
    __syncthreads();
    const int mine = tid < experts ? count[tid] : 0, mt = (mine + bm - 1) / bm;
    start[tid] = mine;
    tile0[tid] = mt;
    for (int d = 1; d < 1024; d <<= 1) { // inclusive scans
        __syncthreads();
        const int a = tid >= d ? start[tid - d] : 0, b = tid >= d ? tile0[tid - d] : 0;
        __syncthreads();
        start[tid] += a;
        tile0[tid] += b;
    }
    __syncthreads();
    const int s0 = start[tid] - mine, t0 = tile0[tid] - mt;
    if (tid == 1023) tiles[0] = tile0[1023];
    for (int j = 0; j < mt; j++) {
        int32_t *e = tiles + 4 + 4 * (t0 + j);
        e[0] = tid;
        e[1] = s0 + j * bm;
        e[2] = s0 + (j + 1) * bm < s0 + mine ? s0 + (j + 1) * bm : s0 + mine;
    }
    count[tid] = s0;
    __syncthreads();
    for (int i = tid; i < n; i += 1024) {
        const int s = atomicAdd(&count[sel[i]], 1);
        slot_of[i] = s;
        src[s] = i / top;
    }
}

// V: f32x4 (widths that are multiples of 4) or float
template <class V>
__global__ void __launch_bounds__(256) combine_kernel(const V *ye, const int32_t *slot_of, const float *wt, int top, int width, V *y, axq_avg avg) {
    const int t = blockIdx.x, e = blockIdx.y * 256 + threadIdx.x; // width, e: in units of V
    if (e >= width) return;
    const size_t i = (size_t)t * width + e;
    V v = y[i];
    for (int j = 0; j < top; j++) v += wt[(size_t)t * top + j] * ye[(size_t)slot_of[(size_t)t * top + j] * width + e];
    y[i] = v;
    if (!avg.out) return;
    const V *past = reinterpret_cast<const V *>(avg.past);
    const size_t stride = avg.stride / (sizeof(V) / 4);
    V s = avg.w[avg.n] * v;
    for (int j = 0; j < avg.n; j++) s += avg.w[j] * past[j * stride + i];
    reinterpret_cast<V *>(avg.out)[i] = s;
}

} // namespace

int axq_moe_route(axq_ctx *ctx, const axq_moe_router &r, const float *z, int ldz, int m, int32_t *sel, float *wt) {
    if (r.experts < 1 || r.experts > AXQ_MOE_MAX_EXPERTS || r.groups < 1 || r.experts % r.groups || r.keep < 1 || r.keep > r.groups || r.top < 1 ||
        r.top > r.keep * (r.experts / r.groups) || m < 1)
        return axq_fail(ctx, AXQ_ERR_SHAPE_MISMATCH, "Shape mismatch: %d of %d experts, from %d of %d groups", r.top, r.experts, r.keep, r.groups);
    if (r.experts <= 64) route_lanes_kernel<<<m, 64, 0, ctx->stream>>>(r, z, ldz, sel, wt);
    else route_kernel<<<m, 64, 0, ctx->stream>>>(r, z, ldz, sel, wt);
    AXQ_LAUNCH_CHECK(ctx, "route_kernel");
    return AXQ_OK;
}

int axq_moe_max_tiles(int n, int experts, int bm) { return n / bm + (experts < n ? experts : n); }

int axq_moe_sort(axq_ctx *ctx, const int32_t *sel, int n, int top, int experts, int bm, int32_t *slot_of, int32_t *src, int32_t *tiles) {
    sort_kernel<<<1, 1024, 0, ctx->stream>>>(sel, n, top, experts, bm, slot_of, src, tiles);
    AXQ_LAUNCH_CHECK(ctx, "sort_kernel");
    return AXQ_OK;
}

int axq_moe_combine(axq_ctx *ctx, const float *ye, const int32_t *slot_of, const float *wt, int top, int m, int width, float *y, const axq_avg &avg) {
    if (width % 4 == 0) // (every row, and avg.stride = m rows, is then a whole number of them)
        combine_kernel<f32x4><<<dim3(m, (width / 4 + 255) / 256), 256, 0, ctx->stream>>>(reinterpret_cast<const f32x4 *>(ye), slot_of, wt, top, width / 4,
                                                                                         reinterpret_cast<f32x4 *>(y), avg);
    else combine_kernel<float><<<dim3(m, (width + 255) / 256), 256, 0, ctx->stream>>>(ye, slot_of, wt, top, width, y, avg);
    AXQ_LAUNCH_CHECK(ctx, "combine_kernel");
    return AXQ_OK;
}
