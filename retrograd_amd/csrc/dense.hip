// Products of bf16 weight matrices held in fragment order (stack_kernels.hpp) with activations in the same order, in
// two arithmetics: bf16 operands on v_mfma_f32_16x16x32_bf16, and f32 activations with the weights widened on
// v_mfma_f32_16x16x4_f32. Rows of the weight are the product's rows (4 consecutive ones per lane), tokens its columns.
#include "dev_common.hpp"
#include "stack_dev.hpp"

namespace rk {

namespace {

struct DenseArgs {
    DenseJob j;
    int T;
    int n_groups;          // row groups of one batch
    int ksplit;            // workgroups that share a row group along K
    float * partial;       // [ksplit][rows padded to 64][N]
    size_t slice;
};

__device__ __forceinline__ void store_out(const DenseOut & o, int arith, int t, int b, int n, int n_end, f4 v) {
    // rows n .. n + 3 of token t (those below n_end are real)
    const int col = o.col0 + b * o.col_batch + n;
    const int cnt = n_end - n < 4 ? n_end - n : 4;
    if (cnt <= 0) return;
    switch (o.kind) {
        case OUT_ACT_RELU2:
#pragma unroll
            for (int i = 0; i < 4; ++i) { const float r = fmaxf(v[i], 0.0f); v[i] = r * r; }
            break;
        case OUT_ACT_GATED: {
            const float g = o.gate[(size_t)t * o.ld_gate + b];
            const float sg = 1.0f / (1.0f + expf(-g));
#pragma unroll
            for (int i = 0; i < 4; ++i) v[i] *= sg;
            break;
        }
        default:
#pragma unroll
            for (int i = 0; i < 4; ++i) v[i] *= o.scale;
    }
    if (o.kind == OUT_F32 || o.kind == OUT_RESIDUAL) {
        float * y = (float *)o.dst + (size_t)t * o.ld + col;
        if (cnt == 4 && (((size_t)t * o.ld + col) & 3) == 0) {
            if (o.kind == OUT_RESIDUAL) v += *(const f4 *)y;
            *(f4 *)y = v;
        } else {
            for (int i = 0; i < cnt; ++i) y[i] = o.kind == OUT_RESIDUAL ? y[i] + v[i] : v[i];
        }
        return;
    }
    if (o.kind == OUT_QUERY) {
        const size_t at = ((size_t)t * o.col_batch + b) * o.ld + n;      // col_batch holds the number of batches here
        if (arith == ARITH_16) {
            __half * q = (__half *)o.dst + at;
            if (cnt == 4) {
                union { __half h[4]; uint2 u; } w;
#pragma unroll
                for (int i = 0; i < 4; ++i) w.h[i] = sat_half(v[i]);
                *(uint2 *)q = w.u;
            } else for (int i = 0; i < cnt; ++i) q[i] = sat_half(v[i]);
        } else {
            float * q = (float *)o.dst + at;
            for (int i = 0; i < cnt; ++i) q[i] = v[i];
        }
        return;
    }
    // activations: four consecutive columns share a group of eight when the first is a multiple of four
    if (arith == ARITH_16) {
        uint16_t * a = (uint16_t *)o.dst;
        if (cnt == 4 && (col & 3) == 0) {
            uint2 u;
            u.x = (uint32_t)bf16_bits(v[0]) | ((uint32_t)bf16_bits(v[1]) << 16);
            u.y = (uint32_t)bf16_bits(v[2]) | ((uint32_t)bf16_bits(v[3]) << 16);
            *(uint2 *)(a + frag_at(t, col, o.ld)) = u;
        } else for (int i = 0; i < cnt; ++i) a[frag_at(t, col + i, o.ld)] = bf16_bits(v[i]);
    } else {
        float * a = (float *)o.dst;
        if (cnt == 4 && (col & 3) == 0) *(f4 *)(a + frag_at(t, col, o.ld)) = v;
        else for (int i = 0; i < cnt; ++i) a[frag_at(t, col + i, o.ld)] = v[i];
    }
}

// Rows tile * 16 + 4 g .. + 3 of token t to the part they belong to.
__device__ __forceinline__ void store_rows(const DenseJob & j, int arith, int t, int b, int tile, int g, const f4 & v) {
    if (tile < j.split_tile) store_out(j.a, arith, t, b, tile * 16 + 4 * g, j.n_a, v);
    else store_out(j.b, arith, t, b, (tile - j.split_tile) * 16 + 4 * g, j.w.n - j.split_tile * 16, v);
}

template <typename TA> struct Operand;      // one lane's eight activation values of a fragment
template <> struct Operand<uint16_t> {
    b8 v;
    __device__ __forceinline__ void load(const uint16_t * p) { v = *(const b8 *)p; }
};
template <> struct Operand<float> {
    f4 a, b;
    __device__ __forceinline__ void load(const float * p) { a = *(const f4 *)p; b = *(const f4 *)(p + 4); }
};
__device__ __forceinline__ void mac(f4 & acc, const b8 & w, const Operand<uint16_t> & x) {
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, x.v, acc, 0, 0, 0);
}
__device__ __forceinline__ void mac(f4 & acc, const b8 & w, const Operand<float> & x) {
    const u4 bits = __builtin_bit_cast(u4, w);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float lo = __builtin_bit_cast(float, bits[i] << 16), hi = __builtin_bit_cast(float, bits[i] & 0xffff0000u);
        const float x0 = i < 2 ? x.a[2 * i] : x.b[2 * i - 4], x1 = i < 2 ? x.a[2 * i + 1] : x.b[2 * i - 3];
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(lo, x0, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(hi, x1, acc, 0, 0, 0);
    }
}

// Operands straight from memory to registers: a wave multiplies RT row tiles with CT token tiles; KW waves of the
// workgroup share the rows and split K, RW sets of them split the rows.
template <typename TA, int RT, int CT, int KW, int RW, bool DUAL>
__global__ __launch_bounds__(64 * KW * RW) void k_dense(DenseArgs A) {
    constexpr int U = sizeof(TA) == 4 ? 2 : (RT * CT >= 8 ? 2 : 4);      // fragments in flight per operand
    const DenseJob & j = A.j;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int kw = wave % KW, rw = wave / KW;
    const int group = blockIdx.x % A.n_groups, ks = blockIdx.x / A.n_groups;
    const int b = blockIdx.z;
    const int tok_tile0 = blockIdx.y * CT;
    const int tile0 = (group * RW + rw) * RT;
    const uint16_t * wbase[RT];
#pragma unroll
    for (int r = 0; r < RT; ++r) {
        const int tile = min(tile0 + r, j.w.tiles - 1);
        wbase[r] = j.w.w + ((size_t)b * j.w.tiles + tile) * (size_t)j.w.kf * 512 + lane * 8;
    }
    f4 acc[RT][CT], done[DUAL ? RT : 1][DUAL ? CT : 1];
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
        for (int c = 0; c < CT; ++c) acc[r][c] = f4{0, 0, 0, 0};
    // this wave's fragments of the whole K
    const int parts = KW * A.ksplit, part = ks * KW + kw;
    const int kf_lo = (int)((int64_t)j.w.kf * part / parts), kf_hi = (int)((int64_t)j.w.kf * (part + 1) / parts);
    auto run = [&](const DenseIn & in, int lo, int hi, int base) {      // fragments [lo, hi), the input's first is `base`
        const TA * xb[CT];
#pragma unroll
        for (int c = 0; c < CT; ++c)
            xb[c] = (const TA *)in.x + ((size_t)(tok_tile0 + c) * in.kf + (size_t)b * in.kf_batch) * 512 + lane * 8 - (ptrdiff_t)base * 512;
        int k = lo;
        for (; k + U <= hi; k += U) {
            b8 w[U][RT];
            Operand<TA> x[U][CT];
#pragma unroll
            for (int u = 0; u < U; ++u) {
#pragma unroll
                for (int r = 0; r < RT; ++r) w[u][r] = *(const b8 *)(wbase[r] + (size_t)(k + u) * 512);
#pragma unroll
                for (int c = 0; c < CT; ++c) x[u][c].load(xb[c] + (size_t)(k + u) * 512);
            }
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int r = 0; r < RT; ++r)
#pragma unroll
                    for (int c = 0; c < CT; ++c) mac(acc[r][c], w[u][r], x[u][c]);
        }
        for (; k < hi; ++k) {
            Operand<TA> x[CT];
#pragma unroll
            for (int c = 0; c < CT; ++c) x[c].load(xb[c] + (size_t)k * 512);
#pragma unroll
            for (int r = 0; r < RT; ++r) {
                const b8 w = *(const b8 *)(wbase[r] + (size_t)k * 512);
#pragma unroll
                for (int c = 0; c < CT; ++c) mac(acc[r][c], w, x[c]);
            }
        }
    };
    auto scale_rows = [&](const float * sc, f4 (&v)[RT][CT]) {
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const int n = (tile0 + r) * 16 + 4 * (lane >> 4);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float f = n + i < j.w.n ? sc[n + i] : 0.0f;
#pragma unroll
                for (int c = 0; c < CT; ++c) v[r][c][i] *= f;
            }
        }
    };
    if constexpr (DUAL) {
        run(j.x, kf_lo, min(kf_hi, j.kf1), 0);
        if (j.scale1) scale_rows(j.scale1, acc);
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
            for (int c = 0; c < CT; ++c) { done[r][c] = acc[r][c]; acc[r][c] = f4{0, 0, 0, 0}; }
        if (j.x2.x) {
            run(j.x2, max(kf_lo, j.kf1), kf_hi, j.kf1);
            if (j.scale2) scale_rows(j.scale2, acc);
        }
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
            for (int c = 0; c < CT; ++c) acc[r][c] += done[r][c];
    } else {
        run(j.x, kf_lo, kf_hi, 0);
    }
    if constexpr (KW > 1) {        // halve the number of partial sums until one is left
        __shared__ f4 red[RW][KW / 2][RT * CT][64];
#pragma unroll
        for (int h = KW / 2; h >= 1; h >>= 1) {
            if (kw >= h && kw < 2 * h)
#pragma unroll
                for (int i = 0; i < RT * CT; ++i) red[rw][kw - h][i][lane] = acc[i / CT][i % CT];
            __syncthreads();
            if (kw < h)
#pragma unroll
                for (int i = 0; i < RT * CT; ++i) acc[i / CT][i % CT] += red[rw][kw][i][lane];
            __syncthreads();
        }
        if (kw != 0) return;
    }
    const int arith = (int)sizeof(TA);
#pragma unroll
    for (int r = 0; r < RT; ++r) {
        const int tile = tile0 + r;
        if (tile >= j.w.tiles) break;
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            const int t = (tok_tile0 + c) * 16 + (lane & 15);
            if (t >= A.T) continue;
            if (A.ksplit > 1) {
                const int n = tile * 16 + 4 * (lane >> 4);
                float * p = A.partial + (size_t)ks * A.slice + (size_t)t * j.w.n + n;
                if (n + 4 <= j.w.n && (j.w.n & 3) == 0) *(f4 *)p = acc[r][c];
                else for (int i = 0; i < 4 && n + i < j.w.n; ++i) p[i] = acc[r][c][i];
            } else {
                store_rows(j, arith, t, b, tile, lane >> 4, acc[r][c]);
            }
        }
    }
}

__global__ void k_dense_pack(const uint16_t * __restrict__ src, int rows, int cols, int64_t rs, int64_t cs,
                             uint16_t * __restrict__ dst, int kf, int row0, int k0) {
    const int64_t n = (int64_t)rows * cols;
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
        const int r = (int)(i / cols), c = (int)(i % cols);
        dst[frag_at(row0 + r, k0 + c, kf)] = src[r * rs + c * cs];
    }
}

template <typename TA, int RT, int CT, int KW, int RW>
void launch(hipStream_t s, DenseArgs & A) {
    const DenseJob & j = A.j;
    A.n_groups = (j.w.tiles + RT * RW - 1) / (RT * RW);
    const dim3 grid((unsigned)(A.n_groups * A.ksplit), (unsigned)((A.T + 16 * CT - 1) / (16 * CT)), (unsigned)j.w.batch);
    if (j.kf1 > 0) hipLaunchKernelGGL((k_dense<TA, RT, CT, KW, RW, true>), grid, dim3(64 * KW * RW), 0, s, A);
    else hipLaunchKernelGGL((k_dense<TA, RT, CT, KW, RW, false>), grid, dim3(64 * KW * RW), 0, s, A);
    check_launch("dense");
}

constexpr int kMaxSlices = 8;
constexpr size_t kSliceFloats = (size_t)64 * 32768;      // tokens x rows of one slice

}  // namespace

void dense_pack(hipStream_t s, const uint16_t * src, int rows, int cols, int64_t row_stride, int64_t k_stride,
                uint16_t * dst, int kf, int row0, int k0) {
    if (rows <= 0 || cols <= 0) return;
    const int64_t n = (int64_t)rows * cols;
    hipLaunchKernelGGL(k_dense_pack, dim3((unsigned)std::min<int64_t>((n + 255) / 256, 8192)), dim3(256), 0, s, src, rows, cols,
                       row_stride, k_stride, dst, kf, row0, k0);
    check_launch("dense_pack");
}

size_t dense_workspace_floats() { return kMaxSlices * kSliceFloats; }

Slices dense(hipStream_t s, int arith, const DenseJob & job, int T, float * ws) {
    Slices out;
    if (T <= 0 || job.w.n <= 0) return out;
    DenseArgs A;
    A.j = job;
    A.T = T;
    A.ksplit = 1;
    A.partial = nullptr;
    A.slice = 0;
    if (A.j.split_tile == 0 && A.j.n_a == 0) { A.j.split_tile = A.j.w.tiles; A.j.n_a = A.j.w.n; }      // one part
    if (arith == ARITH_32) {
        if (T <= 16) launch<float, 1, 1, 4, 1>(s, A);
        else launch<float, 2, 4, 1, 4>(s, A);
        return out;
    }
    if (T <= 16) launch<uint16_t, 1, 1, 8, 1>(s, A);
    else if (T <= 32) launch<uint16_t, 2, 2, 4, 1>(s, A);
    else launch<uint16_t, 4, 4, 1, 4>(s, A);
    return out;
}

}  // namespace rk
