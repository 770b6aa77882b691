// Device-side helpers of the layer-stack kernels.
#pragma once

#include "dev_common.hpp"
#include "stack_kernels.hpp"

#include <algorithm>

namespace rk {

typedef __bf16 b8 __attribute__((ext_vector_type(8)));

// f32 -> bf16, to nearest, ties to even (NaN stays NaN).
__device__ __forceinline__ uint16_t bf16_bits(float v) { return __builtin_bit_cast(uint16_t, (__bf16)v); }
__device__ __forceinline__ float bf16_float(uint16_t b) { return __builtin_bit_cast(float, (uint32_t)b << 16); }

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// Element (row, k) of a buffer in fragment order with kf fragments per row tile.
__device__ __forceinline__ size_t frag_at(int row, int k, int kf) {
    return ((size_t)(row >> 4) * kf + (k >> 5)) * 512 + ((((k >> 3) & 3) * 16 + (row & 15)) * 8) + (k & 7);
}

// Eight consecutive values of a row (k a multiple of 8) as activations of either arithmetic, from element `at` of act on.
template <int ARITH> __device__ __forceinline__ void store_act8_at(void * act, size_t at, const float (&v)[8]) {
    if constexpr (ARITH == ARITH_16) {
        u4 u;
#pragma unroll
        for (int i = 0; i < 4; ++i) u[i] = (uint32_t)bf16_bits(v[2 * i]) | ((uint32_t)bf16_bits(v[2 * i + 1]) << 16);
        *(u4 *)((uint16_t *)act + at) = u;
    } else {
        float * p = (float *)act + at;
        *(f4 *)p = f4{v[0], v[1], v[2], v[3]};
        *(f4 *)(p + 4) = f4{v[4], v[5], v[6], v[7]};
    }
}

template <int ARITH> __device__ __forceinline__ void store_frag8(void * act, int kf, int row, int k, const float (&v)[8]) {
    store_act8_at<ARITH>(act, frag_at(row, k, kf), v);
}

// Element offset inside a cache page of column c of token t (both within the page).
__device__ __forceinline__ size_t cache_at(int t, int c) {
    return ((size_t)(c >> 5) * 2 + (t >> 4)) * 512 + ((((c >> 3) & 3) * 16 + (t & 15)) * 8) + (c & 7);
}

// Sum over the workgroup (any whole number of waves, at most 16), the result in every thread.
__device__ __forceinline__ float block_sum(float v, float * scratch) {
    v = wave_sum(v);
    const int wave = threadIdx.x >> 6, n = (blockDim.x + 63) >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[wave] = v;
    __syncthreads();
    float s = 0.0f;
    for (int i = 0; i < n; ++i) s += scratch[i];
    return s;
}

}  // namespace rk
