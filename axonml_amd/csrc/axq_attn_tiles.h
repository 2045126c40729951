// What the attention kernels of described layers share: the layout of their f16 caches and of matrix-pipe tiles.
//
// Cache in f16: keys [kv_head][position][DP] (head size padded with zeros to 64, 128 or 256), values transposed,
// [kv_head][DVP][position] with positions 4..7 and 8..11 of every 16 exchanged (value_slot), so that both operands of a
// matrix-pipe tile are 16 contiguous bytes per lane.  In f32: keys and values row-major, products on the vector ALU.
#pragma once
#include <hip/hip_fp16.h>

#include "axq_dense.h"

namespace {

typedef _Float16 half8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef const __attribute__((address_space(1))) void gbl_void;
typedef __attribute__((address_space(3))) void lds_void;

constexpr int CHUNK = 64;          // positions per workgroup of a decode step
constexpr float PSCALE = 32768.0f; // weights enter the second product as f16 times this: (0, 1] stays normal down to 2^-29

inline int pad_dim(int d) { return d <= 64 ? 64 : (d <= 128 ? 128 : 256); }
inline int pad_cap(int cap) { return (cap + 63) / 64 * 64; }

__device__ inline _Float16 to_half(float f) { return (_Float16)fminf(fmaxf(f, -65504.f), 65504.f); }

// Where position p of a value row lies: bits 2 and 3 exchanged.
__device__ inline int value_slot(int p) { return (p & ~12) | ((p & 4) << 1) | ((p & 8) >> 1); }

// Row of a 32 x 32 accumulator's register r.
__device__ inline int acc_row(int r, int lane) { return 8 * (r >> 2) + 4 * (lane >> 5) + (r & 3); }

// Values of a prompt's rows into the transposed f16 cache through LDS: grid (32-position tiles, 32-element tiles, kv
// heads) of 256 threads, so that both sides are runs of 64 bytes or more.
__device__ inline void append_values(const float *v, int ldv, int vdim, int m, int pos0, void *vc, int dvp, int capp) {
    __shared__ float tile[32][33];
    const int t0 = blockIdx.x * 32, e0 = blockIdx.y * 32, h = blockIdx.z, x = threadIdx.x & 31, y = threadIdx.x >> 5;
    for (int i = y; i < 32; i += 8)
        tile[i][x] = (t0 + i < m && e0 + x < vdim) ? v[(size_t)(t0 + i) * ldv + (size_t)h * vdim + e0 + x] : 0.f;
    __syncthreads();
    _Float16 *o = reinterpret_cast<_Float16 *>(vc) + (size_t)h * dvp * capp;
    for (int i = y; i < 32; i += 8)
        if (e0 + i < vdim && t0 + x < m) o[(size_t)(e0 + i) * capp + value_slot(pos0 + t0 + x)] = to_half(tile[x][i]);
}

} // namespace
