// Row norms of layer-stack models: the residual stream (completed with the slices the products before left) through an
// RMS or layer norm into activations. Statistics in f32, two passes over the row held in LDS.
#include "stack_dev.hpp"

namespace rk {

namespace {

// VEC: rows of whole groups of four, read and written as such; the slices of a group are all requested at once.
template <int ARITH, int KIND, bool VEC>
__global__ __launch_bounds__(1024) void k_norm_act(float * __restrict__ x, const float * __restrict__ w, int E, float eps,
                                                   const int32_t * __restrict__ rows, void * __restrict__ act, int kf, Slices add,
                                                   const float * __restrict__ plus, void * __restrict__ act_rows) {
    extern __shared__ __attribute__((aligned(16))) float row[];
    __shared__ float scratch[16];
    const int t = rows ? rows[blockIdx.x] : (int)blockIdx.x, n_thr = blockDim.x;
    float * xr = x + (size_t)t * E;
    float sum = 0.0f;
    if constexpr (VEC) {
        for (int k = 4 * (int)threadIdx.x; k < E; k += 4 * n_thr) {
            f4 v = *(const f4 *)(xr + k);
            if (add.n > 0 || plus) {
                f4 s = {0, 0, 0, 0};
                if (plus) s = *(const f4 *)(plus + (size_t)t * E + k);
                for (int base = 0; base < add.n; base += 8) {
                    const float * from = add.data + (size_t)base * add.stride + (size_t)t * E + k;
                    const int n = add.n - base;
                    f4 d[8];
#pragma unroll
                    for (int i = 0; i < 8; ++i) if (i < n) d[i] = *(const f4 *)(from + (size_t)i * add.stride);
#pragma unroll
                    for (int i = 0; i < 8; ++i) if (i < n) s += d[i];
                }
                v += s;
                *(f4 *)(xr + k) = v;
            }
            *(f4 *)(row + k) = v;
            sum += KIND == NORM_LAYER ? v[0] + v[1] + v[2] + v[3] : v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
    } else {
        for (int k = threadIdx.x; k < E; k += n_thr) {
            float v = xr[k];
            if (add.n > 0 || plus) {
                float d = plus ? plus[(size_t)t * E + k] : 0.0f;
                for (int i = 0; i < add.n; ++i) d += add.data[(size_t)i * add.stride + (size_t)t * E + k];
                v += d;
                xr[k] = v;
            }
            row[k] = v;
            sum += KIND == NORM_LAYER ? v : v * v;
        }
    }
    sum = block_sum(sum, scratch);
    float mean = 0.0f;
    if constexpr (KIND == NORM_LAYER) {
        mean = sum / (float)E;
        float q = 0.0f;
        for (int k = threadIdx.x; k < E; k += n_thr) { const float d = row[k] - mean; q += d * d; }
        sum = block_sum(q, scratch);
    }
    const float inv = 1.0f / sqrtf(sum / (float)E + eps);
    for (int k = 8 * (int)threadIdx.x; k < E; k += 8 * n_thr) {
        float v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = k + i < E ? (row[k + i] - mean) * inv * w[k + i] : 0.0f;
        store_frag8<ARITH>(act, kf, blockIdx.x, k, v);
        if (act_rows) store_act8_at<ARITH>(act_rows, (size_t)blockIdx.x * kf * 32 + k, v);
    }
}

__global__ void k_add_slices(float * __restrict__ x, size_t n, Slices add) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
        float d = 0.0f;
        for (int k = 0; k < add.n; ++k) d += add.data[(size_t)k * add.stride + i];
        x[i] += d;
    }
}

}  // namespace

void norm_act(hipStream_t s, int arith, int kind, float * x, const float * w, int E, float eps, const int32_t * rows,
              int n_rows, void * act, int act_kf, const Slices & add, const float * plus, void * act_rows) {
    if (n_rows <= 0) return;
    const size_t lds = (size_t)E * 4;
    const bool vec = E % 4 == 0;
    const dim3 grid((unsigned)n_rows), block(n_rows <= 512 && E >= 2048 ? 1024 : 256);
    auto go = [&](auto kernel) { hipLaunchKernelGGL(kernel, grid, block, lds, s, x, w, E, eps, rows, act, act_kf, add, plus, act_rows); };
    if (arith == ARITH_16) {
        if (kind == NORM_LAYER) vec ? go(k_norm_act<ARITH_16, NORM_LAYER, true>) : go(k_norm_act<ARITH_16, NORM_LAYER, false>);
        else vec ? go(k_norm_act<ARITH_16, NORM_RMS, true>) : go(k_norm_act<ARITH_16, NORM_RMS, false>);
    } else {
        if (kind == NORM_LAYER) vec ? go(k_norm_act<ARITH_32, NORM_LAYER, true>) : go(k_norm_act<ARITH_32, NORM_LAYER, false>);
        else vec ? go(k_norm_act<ARITH_32, NORM_RMS, true>) : go(k_norm_act<ARITH_32, NORM_RMS, false>);
    }
    check_launch("norm_act");
}

void add_slices(hipStream_t s, float * x, int E, int T, const Slices & add) {
    if (add.n <= 0 || T <= 0) return;
    const size_t n = (size_t)T * E;
    hipLaunchKernelGGL(k_add_slices, dim3((unsigned)std::min<size_t>((n + 255) / 256, 4096)), dim3(256), 0, s, x, n, add);
    check_launch("add_slices");
}

}  // namespace rk
