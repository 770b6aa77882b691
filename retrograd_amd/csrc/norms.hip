// Row norms of layer-stack models: the residual stream (completed with the slices the products before left), or what a
// sublayer reads of several residual streams, through an RMS or layer norm into activations. Statistics in f32, two passes
// over the row held in LDS. Also the rows that start a stream.
#include "stack_dev.hpp"

#include <type_traits>

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

// Columns k .. k + W - 1 of row t: the streams take in y by `done` and come back in v, and what the next sublayer reads of
// them. N: streams in registers, the first x.n of them real.
template <int N, int W> struct StreamColumns {
    typedef float vec __attribute__((ext_vector_type(W)));
    vec v[N];
    __device__ __forceinline__ void update(const Streams & x, const float * done, const Slices & y, size_t at) {
#pragma unroll
        for (int a = 0; a < N; ++a)
            if (a < x.n) v[a] = *(const vec *)(x.x + (size_t)a * x.stride + at);
        if (!done) return;
        vec d = vec(0.0f);
        for (int base = 0; base < y.n; base += 8) {
            const float * from = y.data + (size_t)base * y.stride + at;
            const int n = y.n - base;
            vec part[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) if (i < n) part[i] = *(const vec *)(from + (size_t)i * y.stride);
#pragma unroll
            for (int i = 0; i < 8; ++i) if (i < n) d += part[i];
        }
        const float * out = done + x.n, * mix = done + 2 * x.n;
        vec u[N];
#pragma unroll
        for (int b = 0; b < N; ++b) {
            if (b < x.n) {
                u[b] = out[b] * d;
#pragma unroll
                for (int a = 0; a < N; ++a) if (a < x.n) u[b] += mix[a * x.n + b] * v[a];
            }
        }
#pragma unroll
        for (int b = 0; b < N; ++b) if (b < x.n) v[b] = u[b];
    }
    __device__ __forceinline__ vec read(const Streams & x, const float * next) const {
        vec u = vec(0.0f);
#pragma unroll
        for (int a = 0; a < N; ++a) if (a < x.n) u += (next ? next[a] : 1.0f) * v[a];
        return u;
    }
};

template <int ARITH, int N, int W>
__global__ __launch_bounds__(1024) void k_streams_norm_act(Streams x, const float * __restrict__ done, Slices y, const float * __restrict__ next,
                                                           const float * __restrict__ w, int E, float eps, const int32_t * __restrict__ rows,
                                                           void * __restrict__ act, int kf, void * __restrict__ act_rows) {
    extern __shared__ __attribute__((aligned(16))) float row[];
    __shared__ float scratch[16];
    using Columns = StreamColumns<N, W>;
    const int t = rows ? rows[blockIdx.x] : (int)blockIdx.x, n_thr = blockDim.x;
    float sum = 0.0f;
    for (int k = W * (int)threadIdx.x; k < E; k += W * n_thr) {
        const size_t at = (size_t)t * E + k;
        Columns c;
        c.update(x, done, y, at);
        if (done && !rows)
#pragma unroll
            for (int a = 0; a < N; ++a) if (a < x.n) *(typename Columns::vec *)(x.x + (size_t)a * x.stride + at) = c.v[a];
        const typename Columns::vec u = c.read(x, next);
        *(typename Columns::vec *)(row + k) = u;
#pragma unroll
        for (int i = 0; i < W; ++i) sum += u[i] * u[i];
    }
    sum = block_sum(sum, scratch);
    const float inv = 1.0f / sqrtf(sum / (float)E + eps);
    for (int k = 8 * (int)threadIdx.x; k < E; k += 8 * n_thr) {
        float v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = k + i < E ? row[k + i] * inv * w[k + i] : 0.0f;
        store_frag8<ARITH>(act, kf, blockIdx.x, k, v);
        if (act_rows) store_act8_at<ARITH>(act_rows, (size_t)blockIdx.x * kf * 32 + k, v);
    }
}

template <int N> __global__ void k_streams_sum(Streams x, const float * __restrict__ done, Slices y, size_t n, float * __restrict__ out) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
        StreamColumns<N, 1> c;
        c.update(x, done, y, i);
        out[i] = c.read(x, nullptr)[0];
    }
}

__global__ void k_embed_rows(const uint16_t * __restrict__ embed, const int32_t * __restrict__ tok, int E, float scale, size_t n,
                             float * __restrict__ x, int copies, size_t stride) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
        const size_t t = i / E;
        const float v = bf16_float(embed[(size_t)tok[t] * E + (i - t * E)]) * scale;
        for (int a = 0; a < copies; ++a) x[(size_t)a * stride + i] = v;
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

void streams_norm_act(hipStream_t s, int arith, const Streams & x, const float * done, const Slices & y, const float * next,
                      const float * w, int E, float eps, const int32_t * rows, int n_rows, void * act, int act_kf, void * act_rows) {
    if (n_rows <= 0) return;
    if (x.n < 1 || x.n > MAX_STREAMS) throw std::runtime_error("residual streams: more than are supported");
    const dim3 grid((unsigned)n_rows), block(n_rows <= 512 && E >= 2048 ? 1024 : 256);
    auto go = [&](auto kernel) {
        hipLaunchKernelGGL(kernel, grid, block, (size_t)E * 4, s, x, done, y, next, w, E, eps, rows, act, act_kf, act_rows);
    };
    auto width = [&](auto arithmetic, auto n) {
        constexpr int A = decltype(arithmetic)::value, N = decltype(n)::value;
        E % 4 == 0 ? go(k_streams_norm_act<A, N, 4>) : go(k_streams_norm_act<A, N, 1>);
    };
    auto count = [&](auto arithmetic) {
        if (x.n <= 2) width(arithmetic, std::integral_constant<int, 2>());
        else if (x.n == 3) width(arithmetic, std::integral_constant<int, 3>());
        else if (x.n == 4) width(arithmetic, std::integral_constant<int, 4>());
        else width(arithmetic, std::integral_constant<int, MAX_STREAMS>());
    };
    if (arith == ARITH_16) count(std::integral_constant<int, ARITH_16>());
    else count(std::integral_constant<int, ARITH_32>());
    check_launch("streams_norm_act");
}

void streams_sum(hipStream_t s, const Streams & x, const float * done, const Slices & y, int E, int T, float * out) {
    if (T <= 0) return;
    if (x.n < 1 || x.n > MAX_STREAMS) throw std::runtime_error("residual streams: more than are supported");
    const size_t n = (size_t)T * E;
    hipLaunchKernelGGL(k_streams_sum<MAX_STREAMS>, dim3((unsigned)std::min<size_t>((n + 255) / 256, 4096)), dim3(256), 0, s, x, done, y, n, out);
    check_launch("streams_sum");
}

void embed_rows(hipStream_t s, const uint16_t * embed, const int32_t * tok, int E, float scale, int T, float * x, int copies, size_t stride) {
    if (T <= 0) return;
    const size_t n = (size_t)T * E;
    hipLaunchKernelGGL(k_embed_rows, dim3((unsigned)std::min<size_t>((n + 255) / 256, 8192)), dim3(256), 0, s, embed, tok, E, scale, n, x, copies, stride);
    check_launch("embed_rows");
}

void add_slices(hipStream_t s, float * x, int E, int T, const Slices & add) {
    if (add.n <= 0 || T <= 0) return;
    const size_t n = (size_t)T * E;
    hipLaunchKernelGGL(k_add_slices, dim3((unsigned)std::min<size_t>((n + 255) / 256, 4096)), dim3(256), 0, s, x, n, add);
    check_launch("add_slices");
}

}  // namespace rk
