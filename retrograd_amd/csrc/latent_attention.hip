// Latent attention: keys and values of every head are up-projections of one cached latent per token, so a query is
// absorbed into the latent space first (q' = W_uk^T q) and every head attends over the same cached rows, with a
// sliding window. The attended latents leave as activations for the value up-projection.
#include "stack_dev.hpp"

namespace rk {

namespace {

template <typename EL> __device__ __forceinline__ float el_float(EL v);
template <> __device__ __forceinline__ float el_float<__half>(__half v) { return __half2float(v); }
template <> __device__ __forceinline__ float el_float<float>(float v) { return v; }
template <typename EL> __device__ __forceinline__ EL float_el(float v);
template <> __device__ __forceinline__ __half float_el<__half>(float v) { return sat_half(v); }
template <> __device__ __forceinline__ float float_el<float>(float v) { return v; }

// One wave per token and norm: the queries' latent, and (blockIdx.y = 1) the latent that goes into the cache.
template <int ARITH>
__global__ __launch_bounds__(64) void k_latent_norms(LatentNorms a) {
    using EL = typename std::conditional<ARITH == ARITH_16, __half, float>::type;
    const int t = blockIdx.x, lane = threadIdx.x;
    const bool kv = blockIdx.y == 1;
    const int n = kv ? a.kv_rank : a.q_rank;
    const float * src = a.proj + (size_t)t * a.ld + (kv ? a.kv_col : 0);
    const float * w = kv ? a.kv_w : a.q_w;
    float q = 0.0f;
    for (int k = lane; k < n; k += 64) q += src[k] * src[k];
    q = wave_sum(q);
    const float inv = 1.0f / sqrtf(q / (float)n + a.eps);
    const int cell = kv ? a.cell[t] : 0;
    EL * page = kv ? (EL *)a.pool + (size_t)(cell / PAGE) * latent_page_elems(a.pool_kf) : nullptr;
    const int padded = (n + 31) / 32 * 32;
    for (int k = 8 * lane; k < padded; k += 512) {
        float v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = k + i < n ? src[k + i] * inv * w[k + i] : 0.0f;
        if (kv) {
            EL * dst = page + latent_at(cell % PAGE, k);
#pragma unroll
            for (int i = 0; i < 8; ++i) dst[i] = float_el<EL>(v[i]);
        } else {
            store_frag8<ARITH>(a.act_q, a.act_q_kf, t, k, v);
        }
    }
}

// Any rank, either element type: one workgroup per query column, keys in batches of one per thread, f32 throughout.
template <int ARITH>
__global__ __launch_bounds__(256) void k_latent_attention_any(LatentAttn a) {
    using EL = typename std::conditional<ARITH == ARITH_16, __half, float>::type;
    extern __shared__ float sm[];
    const int R = a.kf * 32;
    float * q = sm, * p = sm + R;             // [R], [256]
    __shared__ float scratch[16];
    const LatentBlock blk = a.blocks[blockIdx.x];
    const RowDesc row = a.rows[blk.row];
    const int n_cols = row.n * a.H;
    const size_t page_elems = latent_page_elems(a.kf);
    for (int c = blk.col0; c < min(blk.col0 + a.block_cols, n_cols); ++c) {
        const int tok = c / a.H, h = c % a.H, t = row.tok_off + tok, pos = row.pos0 + tok;
        const int lo = a.window > 0 ? max(row.kv_begin, pos - a.window + 1) : row.kv_begin;
        const EL * qr = (const EL *)a.q + ((size_t)t * a.H + h) * R;
        __syncthreads();
        for (int k = threadIdx.x; k < R; k += 256) q[k] = el_float<EL>(qr[k]);
        float m = -INFINITY, l = 0.0f;
        float acc[4] = {0, 0, 0, 0};                                      // columns threadIdx.x + 256 i
        for (int base = lo; base <= pos; base += 256) {
            __syncthreads();
            const int key = base + threadIdx.x;
            float s = -INFINITY;
            if (key <= pos) {
                const int pg = a.table[(size_t)row.slot * a.max_pages + key / PAGE];
                const EL * page = (const EL *)a.pool + (size_t)pg * page_elems;
                s = 0.0f;
                for (int k = 0; k < R; k += 8) {
                    const EL * e = page + latent_at(key % PAGE, k);
#pragma unroll
                    for (int i = 0; i < 8; ++i) s += q[k + i] * el_float<EL>(e[i]);
                }
            }
            float bm = s;
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) bm = fmaxf(bm, __shfl_xor(bm, o, 64));
            if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = bm;
            __syncthreads();
            bm = fmaxf(fmaxf(scratch[0], scratch[1]), fmaxf(scratch[2], scratch[3]));
            const float m2 = fmaxf(m, bm), f = exp2f(m - m2);
            p[threadIdx.x] = exp2f(s - m2);
            const float bl = block_sum(p[threadIdx.x], scratch);          // also orders the writes to p
            l = l * f + bl;
            m = m2;
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] *= f;
            const int n = min(256, pos - base + 1);
            for (int k = 0; k < n; ++k) {
                const int kk = base + k;
                const int pg = a.table[(size_t)row.slot * a.max_pages + kk / PAGE];
                const EL * page = (const EL *)a.pool + (size_t)pg * page_elems;
                const float pk = p[k];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int col = threadIdx.x + 256 * i;
                    if (col < R) acc[i] += pk * el_float<EL>(page[latent_at(kk % PAGE, col)]);
                }
            }
        }
        const float inv = 1.0f / l;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int col = threadIdx.x + 256 * i;
            if (col >= R) break;
            const size_t at = frag_at(t, h * R + col, a.out_kf);
            if constexpr (ARITH == ARITH_16) ((uint16_t *)a.out)[at] = bf16_bits(acc[i] * inv);
            else ((float *)a.out)[at] = acc[i] * inv;
        }
    }
}

__global__ void k_copy16(const u4 * __restrict__ src, u4 * __restrict__ dst, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) dst[i] = src[i];
}
__global__ void k_copy4(const float * __restrict__ src, float * __restrict__ dst, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) dst[i] = src[i];
}

// rows[i][c] <-> column c of cell cells[i]; a column group of eight per thread.
template <typename EL>
__global__ void k_latent_cells(EL * __restrict__ pool, int kf, const int32_t * __restrict__ cells, int n, EL * __restrict__ rows, bool gather) {
    const int groups = kf * 4;
    const int64_t total = (int64_t)n * groups;
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (int64_t)gridDim.x * blockDim.x) {
        const int r = (int)(i / groups), c = (int)(i % groups) * 8;
        const int cell = cells[r];
        EL * p = pool + (size_t)(cell / PAGE) * latent_page_elems(kf) + latent_at(cell % PAGE, c);
        EL * o = rows + (size_t)r * kf * 32 + c;
#pragma unroll
        for (int k = 0; k < 8; ++k) { if (gather) o[k] = p[k]; else p[k] = o[k]; }
    }
}

}  // namespace

void latent_norms(hipStream_t s, int arith, const LatentNorms & a, int T) {
    if (T <= 0) return;
    const dim3 grid((unsigned)T, a.kv_w ? 2u : 1u);
    if (arith == ARITH_16) hipLaunchKernelGGL(k_latent_norms<ARITH_16>, grid, dim3(64), 0, s, a);
    else hipLaunchKernelGGL(k_latent_norms<ARITH_32>, grid, dim3(64), 0, s, a);
    check_launch("latent_norms");
}

int latent_block_cols(int arith, int H, int n_tokens, int n_rows) { return 1; }
int latent_splits(int arith, const LatentAttn & a, int max_resident) { return 1; }
size_t latent_partial_floats(int T, int H, int kf, int splits) { return splits > 1 ? (size_t)T * H * splits * (kf * 32 + 2) : 0; }

void latent_attention(hipStream_t s, int arith, const LatentAttn & a, int T) {
    if (a.n_blocks <= 0) return;
    if (a.kf * 32 > 1024) throw std::runtime_error("latent attention: latents of at most 1024 columns");
    const size_t lds = ((size_t)a.kf * 32 + 256) * 4;
    const dim3 grid((unsigned)a.n_blocks);
    if (arith == ARITH_16) hipLaunchKernelGGL(k_latent_attention_any<ARITH_16>, grid, dim3(256), lds, s, a);
    else hipLaunchKernelGGL(k_latent_attention_any<ARITH_32>, grid, dim3(256), lds, s, a);
    check_launch("latent_attention");
}

void latent_copy_page(hipStream_t s, void * pool, size_t page_bytes, int src, int dst) {
    const size_t n = page_bytes / 16;
    hipLaunchKernelGGL(k_copy16, dim3((unsigned)std::min<size_t>((n + 255) / 256, 256)), dim3(256), 0, s,
                       (const u4 *)((const uint8_t *)pool + (size_t)src * page_bytes), (u4 *)((uint8_t *)pool + (size_t)dst * page_bytes), n);
    check_launch("latent_copy_page");
}

void copy_floats(hipStream_t s, const float * src, float * dst, size_t n) {
    if (n == 0) return;
    hipLaunchKernelGGL(k_copy4, dim3((unsigned)std::min<size_t>((n + 255) / 256, 1024)), dim3(256), 0, s, src, dst, n);
    check_launch("copy_floats");
}

void latent_cells(hipStream_t s, void * pool, int kf, int elem, const int32_t * cells, int n, void * rows, bool gather) {
    if (n <= 0) return;
    const int64_t total = (int64_t)n * kf * 4;
    const dim3 grid((unsigned)std::min<int64_t>((total + 255) / 256, 4096));
    if (elem == 2) hipLaunchKernelGGL(k_latent_cells<uint16_t>, grid, dim3(256), 0, s, (uint16_t *)pool, kf, cells, n, (uint16_t *)rows, gather);
    else hipLaunchKernelGGL(k_latent_cells<uint32_t>, grid, dim3(256), 0, s, (uint32_t *)pool, kf, cells, n, (uint32_t *)rows, gather);
    check_launch("latent_cells");
}

}  // namespace rk
