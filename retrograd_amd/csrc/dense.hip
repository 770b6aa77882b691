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
    float * partial;       // [ksplit][T][N]: the product leaves its K-slices here (null: it goes to its outputs)
    size_t slice;
    int grid_k;            // workgroups of one K-slice (the LDS kernel)
    ExpertGroups groups;
};

// Slots of an expert product's tile (a plain product: its tokens), and whose row the lane reads of slot `slot`.
struct Columns { int b, first, end; };
template <bool GROUPED> __device__ __forceinline__ bool columns_of(const DenseArgs & A, int tile, Columns & c) {
    if constexpr (GROUPED) {
        if (tile >= *A.groups.n_tiles) return false;
        const int4 e = ((const int4 *)A.groups.tiles)[tile];
        c = {e.x, e.y, e.y + e.z};
    }
    return true;
}
template <bool GROUPED> __device__ __forceinline__ int row_of(const DenseArgs & A, const Columns & c, int slot) {
    if constexpr (GROUPED) {
        if (A.j.gather) return A.groups.slot_pair[min(slot, c.end - 1)] / A.groups.top;
    }
    return slot;
}

// Four columns n .. n + 3 of token t: two pairs of one head.
template <int ARITH> __device__ __forceinline__ void store_rotary(const DenseOut & o, int t, int n, f4 v) {
    using EL = typename std::conditional<ARITH == ARITH_16, __half, float>::type;
    const RotaryOut & r = o.rot;
    auto put = [](EL * dst, const f4 & u) {
        if constexpr (ARITH == ARITH_16) {
            union { __half h[4]; uint2 w; } p;
#pragma unroll
            for (int i = 0; i < 4; ++i) p.h[i] = sat_half(u[i]);
            *(uint2 *)dst = p.w;
        } else {
            *(f4 *)dst = u;
        }
    };
    const int own = n - (r.H + r.G) * r.kf * 32;         // column of the values' own rows
    if (own >= 0) {
        const int cell = r.cell[t];
        put((EL *)r.v_pool + (size_t)(cell / PAGE) * cache_page_elems(r.vf * r.G) + cache_at(cell % PAGE, own), v);
        return;
    }
    const int head = n / (r.kf * 32), c = n - head * r.kf * 32;
    f4 y = v;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int pair = (c >> 1) + i;
        if (pair < r.pairs) {
            const float2 cs = *(const float2 *)(r.table + 2 * ((size_t)t * r.pairs + pair));
            y[2 * i] = v[2 * i] * cs.x - v[2 * i + 1] * cs.y;
            y[2 * i + 1] = v[2 * i + 1] * cs.x + v[2 * i] * cs.y;
        }
    }
    if (head < r.H) {
        put((EL *)o.dst + ((size_t)t * r.H + head) * (r.kf * 32) + c, y);
    } else {
        const int cell = r.cell[t];
        const size_t at = (size_t)(cell / PAGE) * cache_page_elems(r.kf * r.G) + cache_at(cell % PAGE, (head - r.H) * r.kf * 32 + c);
        put((EL *)r.k_pool + at, y);
        if (r.vf == 0) put((EL *)r.v_pool + at, v);
    }
}

// gate and up of the same four columns
template <int KIND> __device__ __forceinline__ f4 glu(const DenseOut & o, const f4 & gate, const f4 & up) {
    f4 v;
    if constexpr (KIND == OUT_ACT_CLAMPED) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float g = fminf(gate[i], o.limit), u = fminf(fmaxf(up[i], -o.limit), o.limit);
            v[i] = g / (1.0f + expf(-o.slope * g)) * (u + 1.0f);
        }
        return v;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float z = gate[i];
        // 0.5 (1 + tanh(u)) = sigmoid(2 u)
        const float u = KIND == OUT_ACT_GEGLU ? 1.5957691216057308f * (z + 0.044715f * z * z * z) : z;
        v[i] = z / (1.0f + expf(-u)) * up[i];
    }
    return v;
}

// One compiled form per pair of output kinds (part a, part b): a kernel that chose among all of them at run time would
// spend more on fetching its epilogue's instructions than on a product of a few hundred columns.
template <int KIND, int ARITH>
__device__ __forceinline__ void store_out(const DenseOut & o, int t, int b, int n, int n_end, f4 v) {
    // rows n .. n + 3 of token t (those below n_end are real)
    const int cnt = n_end - n;
    if (cnt <= 0) return;
    if constexpr (KIND == OUT_ROTARY) {
        store_rotary<ARITH>(o, t, n, v);
        return;
    }
    if constexpr (KIND == OUT_ACT_RELU2) {
#pragma unroll
        for (int i = 0; i < 4; ++i) { const float r = fmaxf(v[i], 0.0f); v[i] = r * r; }
    } else if constexpr (KIND == OUT_ACT_GATED) {
        v *= 1.0f / (1.0f + expf(-o.gate[(size_t)t * o.ld_gate + b]));
    } else if constexpr (KIND == OUT_F32_CAPPED) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = o.limit * tanhf(v[i] / o.limit);
    } else if constexpr (KIND != OUT_RESIDUAL && !out_is_glu(KIND) && KIND != OUT_EXPERT) {
        v *= o.scale;
    }
    const int col = o.col0 + (KIND == OUT_QUERY ? 0 : b * o.col_batch) + n;
    if constexpr (KIND == OUT_F32 || KIND == OUT_F32_CAPPED || KIND == OUT_RESIDUAL) {
        const size_t at = (size_t)t * o.ld + col;
        float * y = (float *)o.dst + at;
        if (cnt >= 4 && (at & 3) == 0) {
            if constexpr (KIND == OUT_RESIDUAL) v += *(const f4 *)y;
            *(f4 *)y = v;
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) if (i < cnt) y[i] = KIND == OUT_RESIDUAL ? y[i] + v[i] : v[i];
        }
    } else if constexpr (KIND == OUT_QUERY) {
        const size_t at = ((size_t)t * o.col_batch + b) * o.ld + n;      // col_batch holds the number of batches here
        if constexpr (ARITH == ARITH_16) {                               // whole fragments: n_end and ld are multiples of 32
            union { __half h[4]; uint2 u; } w;
#pragma unroll
            for (int i = 0; i < 4; ++i) w.h[i] = sat_half(v[i]);
            *(uint2 *)((__half *)o.dst + at) = w.u;
        } else {
            *(f4 *)((float *)o.dst + at) = v;
        }
    } else if (cnt >= 4 && (col & 3) == 0) {       // activations: four columns from a multiple of four share a group of eight
        if constexpr (ARITH == ARITH_16) {
            uint2 u;
            u.x = (uint32_t)bf16_bits(v[0]) | ((uint32_t)bf16_bits(v[1]) << 16);
            u.y = (uint32_t)bf16_bits(v[2]) | ((uint32_t)bf16_bits(v[3]) << 16);
            *(uint2 *)((uint16_t *)o.dst + frag_at(t, col, o.ld)) = u;
        } else {
            *(f4 *)((float *)o.dst + frag_at(t, col, o.ld)) = v;
        }
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            if (i >= cnt) break;
            const size_t at = frag_at(t, col + i, o.ld);
            if constexpr (ARITH == ARITH_16) ((uint16_t *)o.dst)[at] = bf16_bits(v[i]);
            else ((float *)o.dst)[at] = v[i];
        }
    }
}

// Rows tile * 16 + 4 g .. + 3 of token t to the part they belong to (KB < 0: there is only part a).
// A gated part is stored at its gate tiles (the even ones of the part, which starts at an even tile): `next` holds the
// rows of the tile behind, its up rows.
template <int KA, int KB, int ARITH>
__device__ __forceinline__ void store_rows(const DenseJob & j, int t, int b, int tile, int g, const f4 & v, const f4 & next) {
    if (KB < 0 || tile < j.split_tile) {
        if constexpr (out_is_glu(KA)) {
            if (tile & 1) return;
            store_out<KA, ARITH>(j.a, t, b, tile * 8 + 4 * g, j.n_a / 2, glu<KA>(j.a, v, next));
        } else {
            store_out<KA, ARITH>(j.a, t, b, tile * 16 + 4 * g, j.n_a, v);
        }
    } else if constexpr (KB >= 0) {
        const int rows = j.w.n - j.split_tile * 16, at = tile - j.split_tile;
        if constexpr (out_is_glu(KB)) {
            if (at & 1) return;
            store_out<KB, ARITH>(j.b, t, b, at * 8 + 4 * g, rows / 2, glu<KB>(j.b, v, next));
        } else {
            store_out<KB, ARITH>(j.b, t, b, at * 16 + 4 * g, rows, v);
        }
    }
}

// An expert's rows of the pair in slot t.
__device__ __forceinline__ void store_expert(const DenseArgs & A, int t, int n, f4 v) {
    const DenseOut & o = A.j.a;
    const int cnt = A.j.w.n - n;
    if (cnt <= 0) return;
    const int pair = A.groups.slot_pair[t], token = pair / A.groups.top, choice = pair - token * A.groups.top;
    if (!A.groups.weigh_input) v *= A.groups.weight[pair];
    float * y = (float *)o.dst + (size_t)choice * o.stride + (size_t)token * o.ld + n;
    if (cnt >= 4 && (o.ld & 3) == 0) *(f4 *)y = v;
    else
        for (int i = 0; i < 4 && i < cnt; ++i) y[i] = v[i];
}

// What an expert's input rows are multiplied with, for the pair in slot t.
__device__ __forceinline__ float input_weight(const DenseArgs & A, int t) {
    return A.groups.weigh_input ? A.groups.weight[A.groups.slot_pair[t]] : 1.0f;
}

// K-slice `ks` of rows n .. n + 3 of token t; `add`: to what is there.
__device__ __forceinline__ void store_slice(const DenseArgs & A, int ks, int t, int n, f4 v, bool add) {
    const int cnt = A.j.w.n - n;
    if (cnt <= 0) return;
    float * p = A.partial + (size_t)ks * A.slice + (size_t)t * A.j.w.n + n;
    if (cnt >= 4 && (A.j.w.n & 3) == 0) {
        if (add) v += *(const f4 *)p;
        *(f4 *)p = v;
    } else {
        for (int i = 0; i < 4 && i < cnt; ++i) p[i] = add ? p[i] + v[i] : v[i];
    }
}

// Biases of rows 4 g .. 4 g + 3 of a tile.
__device__ __forceinline__ f4 bias_of(const DenseJob & j, int b, int tile, int g) {
    return *(const f4 *)(j.bias + ((size_t)b * j.w.tiles + tile) * 16 + 4 * g);
}

__device__ __forceinline__ float token_factor(const DenseJob & j, int t) {
    return j.token_gate ? 1.0f / (1.0f + expf(-j.token_gate[(size_t)t * j.ld_token_gate])) : 1.0f;
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
template <typename TA, int KA, int KB, int RT, int CT, int KW, int RW, bool GROUPED>
__global__ __launch_bounds__(64 * KW * RW) void k_dense(DenseArgs A) {
    constexpr bool DUAL = KA == OUT_RESIDUAL;
    static_assert(RT % 2 == 0 || !(out_is_glu(KA) || out_is_glu(KB)));
    constexpr int U = sizeof(TA) == 4 ? 2 : (RT * CT >= 8 ? 2 : 4);      // fragments in flight per operand
    const DenseJob & j = A.j;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int kw = wave % KW, rw = wave / KW;
    const int group = blockIdx.x % A.n_groups, ks = blockIdx.x / A.n_groups;
    Columns cols = {(int)blockIdx.z, (int)blockIdx.y * CT * 16, A.T};
    if (!columns_of<GROUPED>(A, blockIdx.y, cols)) return;
    const int b = cols.b;
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
        {
            const int row = row_of<GROUPED>(A, cols, cols.first + c * 16 + (lane & 15));
            if (GROUPED && j.gather) xb[c] = (const TA *)in.x + (size_t)row * in.kf * 32 + (lane >> 4) * 8;
            else xb[c] = (const TA *)in.x + ((size_t)(row >> 4) * in.kf + (GROUPED ? 0 : (size_t)b * in.kf_batch)) * 512 + ((lane & 48) | (row & 15)) * 8 - (ptrdiff_t)base * 512;
        }
        const size_t step = GROUPED && j.gather ? 32 : 512;       // elements from one fragment of a row to the next
        int k = lo;
        for (; k + U <= hi; k += U) {
            b8 w[U][RT];
            Operand<TA> x[U][CT];
#pragma unroll
            for (int u = 0; u < U; ++u) {
#pragma unroll
                for (int r = 0; r < RT; ++r) w[u][r] = *(const b8 *)(wbase[r] + (size_t)(k + u) * 512);
#pragma unroll
                for (int c = 0; c < CT; ++c) x[u][c].load(xb[c] + (size_t)(k + u) * step);
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
            for (int c = 0; c < CT; ++c) x[c].load(xb[c] + (size_t)k * step);
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
    constexpr int ARITH = (int)sizeof(TA);
    if constexpr (DUAL) {
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            const float f = token_factor(j, min(cols.first + c * 16 + (lane & 15), cols.end - 1));
#pragma unroll
            for (int r = 0; r < RT; ++r) acc[r][c] *= f;
        }
    }
    if (j.bias && ks == 0) {
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const f4 f = bias_of(j, b, min(tile0 + r, j.w.tiles - 1), lane >> 4);
#pragma unroll
            for (int c = 0; c < CT; ++c) acc[r][c] += f;
        }
    }
#pragma unroll
    for (int r = 0; r < RT; ++r) {
        const int tile = tile0 + r;
        if (tile >= j.w.tiles) break;
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            const int t = cols.first + c * 16 + (lane & 15);
            if (t >= cols.end) continue;
            if constexpr (KA == OUT_EXPERT) {
                store_expert(A, t, tile * 16 + 4 * (lane >> 4), acc[r][c]);
            } else if (DUAL && A.partial) {
                store_slice(A, ks, t, tile * 16 + 4 * (lane >> 4), acc[r][c], false);
            } else {
                f4 v = acc[r][c], next = acc[RT > 1 ? r ^ 1 : r][c];
                if constexpr (GROUPED) {
                    const float f = input_weight(A, t);
                    v *= f;
                    next *= f;
                }
                store_rows<KA, KB, ARITH>(j, t, GROUPED ? 0 : b, tile, lane >> 4, v, next);
            }
        }
    }
}

__global__ void k_dense_pack(const uint16_t * __restrict__ src, int rows, int cols, int64_t rs, int64_t cs,
                             uint16_t * __restrict__ dst, int kf, PackMap row, PackMap col) {
    const int64_t n = (int64_t)rows * cols;
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
        const int r = (int)(i / cols), c = (int)(i % cols);
        dst[frag_at(row.at + r / row.run * row.step + r % row.run, col.at + c / col.run * col.step + c % col.run, kf)] = src[r * rs + c * cs];
    }
}

// Operands through LDS, for steps of many tokens in bf16: a workgroup of four waves owns 32 RT rows x 32 CT tokens, two
// waves along each, a wave RT x CT tiles. Fragments of both operands go to LDS by direct loads in the order they are
// stored in; three buffers, so that two fragments are on their way while one is multiplied. A two-part product adds its
// first part to the residual, then its second.
template <int KA, int KB, int RT, int CT, bool GROUPED>
__global__ __launch_bounds__(256, 2) void k_dense_lds(DenseArgs A, int n_tok_blocks) {
    constexpr bool DUAL = KA == OUT_RESIDUAL;
    constexpr int PIECES = 2 * RT + 2 * CT;                   // KiB of a stage: its row tiles, then its token tiles
    constexpr int PER_WAVE = (PIECES + 3) / 4;
    static_assert(PIECES % 4 == 0);
    __shared__ __attribute__((aligned(16))) uint8_t lds[3][PIECES * 1024];
    const DenseJob & j = A.j;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), wn = wave & 1, wt = wave >> 1;
    // workgroup b runs on XCD b % 8: an XCD takes every eighth row block, and walks eight token blocks per row block, so
    // that its concurrent workgroups share both operands in its L2
    const int n_groups = A.n_groups;
    int gb, tb, ks;
    if constexpr (GROUPED) {           // the row blocks of a tile of slots on one XCD, which keeps the gathered rows in its L2
        const int i = blockIdx.x >> 3;
        gb = i % n_groups;
        tb = (i / n_groups) * 8 + (blockIdx.x & 7);
        ks = 0;
    } else {
        const int b = A.ksplit > 1 ? blockIdx.x % A.grid_k : blockIdx.x;
        ks = A.ksplit > 1 ? blockIdx.x / A.grid_k : 0;
        const int xcd = b & 7, i = b >> 3, per = (n_groups + 7) / 8, group = 8 * per;
        const int band = i / group, r = i - band * group, tn = min(8, n_tok_blocks - band * 8);
        gb = (r / tn) * 8 + xcd;
        tb = band * 8 + r % tn;
        if (gb >= n_groups || tb >= n_tok_blocks || r / tn >= per) return;
    }
    Columns cols = {0, tb * 32 * CT, A.T};
    if (!columns_of<GROUPED>(A, tb, cols)) return;
    const int tile0 = gb * 2 * RT;
    const uint16_t * weights = j.w.w + (size_t)cols.b * j.w.tiles * j.w.kf * 512;
    f4 acc[RT][CT];
    auto clear = [&]() {
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
            for (int c = 0; c < CT; ++c) acc[r][c] = f4{0, 0, 0, 0};
    };
    auto run = [&](const DenseIn & in, int lo, int hi, int base) {
        const int n = hi - lo;
        if (n <= 0) return;
        const uint8_t * src[PER_WAVE];
        uint32_t off[GROUPED ? PER_WAVE : 1];                 // the lane's place: a row of its own where rows are gathered
#pragma unroll
        for (int i = 0; i < PER_WAVE; ++i) {
            const int piece = wave + 4 * i;
            if constexpr (GROUPED) off[i] = (uint32_t)lane * 16;
            if (piece < 2 * RT) src[i] = (const uint8_t *)(weights + ((size_t)min(tile0 + piece, j.w.tiles - 1) * j.w.kf + lo) * 512);
            else if constexpr (GROUPED) {
                // plain rows: four lanes take a row's 64 bytes, dealt so that the reads below meet no bank twice
                src[i] = (const uint8_t *)((const uint16_t *)in.x + (size_t)(lo - base) * (j.gather ? 32 : 512));
                const int row = row_of<GROUPED>(A, cols, cols.first + (piece - 2 * RT) * 16 + (j.gather ? lane >> 2 : lane & 15));
                if (j.gather) off[i] = (uint32_t)row * (uint32_t)in.kf * 64 + (uint32_t)((lane & 3) ^ ((lane >> 4) & 3)) * 16;
                else off[i] = (uint32_t)(row >> 4) * (uint32_t)in.kf * 1024 + (uint32_t)lane * 16;
            } else src[i] = (const uint8_t *)((const uint16_t *)in.x + ((size_t)((cols.first >> 4) + piece - 2 * RT) * in.kf + (lo - base)) * 512);
        }
        const uint32_t to = lds_offset(lds);
        auto stage = [&](int k, int b) {
            const int kk = min(k, n - 1);
#pragma unroll
            for (int i = 0; i < PER_WAVE; ++i)
                lds_dma16(src[i] + (size_t)kk * (GROUPED && wave + 4 * i >= 2 * RT && j.gather ? 64 : 1024), GROUPED ? off[GROUPED ? i : 0] : (uint32_t)lane * 16, to + (uint32_t)(b * PIECES + wave + 4 * i) * 1024);
        };
        const int x_lane = GROUPED && j.gather ? ((lane & 15) * 4 + ((lane >> 4) ^ ((lane >> 2) & 3))) * 16 : lane * 16;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");      // the part before has stored, and the counted waits start at none
        __syncthreads();                                      // the buffers may still be read by the part before
        stage(0, 0);
        stage(1, 1);
        int b = 0;
        for (int k = 0; k < n; ++k) {
            asm volatile("s_waitcnt vmcnt(%0)" :: "n"(PER_WAVE) : "memory");
            __syncthreads();
            stage(k + 2, b == 0 ? 2 : b - 1);
            const uint8_t * cur = lds[b];
            b8 w[RT], x[CT];
#pragma unroll
            for (int r = 0; r < RT; ++r) w[r] = *(const b8 *)(cur + (wn * RT + r) * 1024 + lane * 16);
#pragma unroll
            for (int c = 0; c < CT; ++c) x[c] = *(const b8 *)(cur + (2 * RT + wt * CT + c) * 1024 + x_lane);
#pragma unroll
            for (int r = 0; r < RT; ++r)
#pragma unroll
                for (int c = 0; c < CT; ++c) acc[r][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[r], x[c], acc[r][c], 0, 0, 0);
            b = b == 2 ? 0 : b + 1;
        }
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");      // nothing may land in LDS that another workgroup owns by then
    };
    auto store = [&](const float * scale, bool first) {
        const bool biased = j.bias && ks == 0 && first;
        if (!DUAL && biased) {
#pragma unroll
            for (int r = 0; r < RT; ++r) {
                const f4 f = bias_of(j, cols.b, min(tile0 + wn * RT + r, j.w.tiles - 1), lane >> 4);
#pragma unroll
                for (int c = 0; c < CT; ++c) acc[r][c] += f;
            }
        }
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const int tile = tile0 + wn * RT + r;
            if (tile >= j.w.tiles) break;
            f4 f = {1, 1, 1, 1};
            if (scale) {
                const int n = tile * 16 + 4 * (lane >> 4);
#pragma unroll
                for (int i = 0; i < 4; ++i) f[i] = n + i < j.w.n ? scale[n + i] : 0.0f;
            }
#pragma unroll
            for (int c = 0; c < CT; ++c) {
                const int t = cols.first + (wt * CT + c) * 16 + (lane & 15);
                if (t >= cols.end) continue;
                f4 v = acc[r][c];
                if constexpr (DUAL) {
                    v *= f * token_factor(j, t);
                    if (biased) v += bias_of(j, 0, tile, lane >> 4);
                }
                if constexpr (KA == OUT_EXPERT) {
                    store_expert(A, t, tile * 16 + 4 * (lane >> 4), v);
                } else if (DUAL && A.partial) {
                    store_slice(A, ks, t, tile * 16 + 4 * (lane >> 4), v, !first);
                } else {
                    f4 next = acc[r ^ 1][c];
                    if constexpr (GROUPED) {
                        const float w = input_weight(A, t);
                        v *= w;
                        next *= w;
                    }
                    store_rows<KA, KB, ARITH_16>(j, t, 0, tile, lane >> 4, v, next);
                }
            }
        }
    };
    clear();
    if constexpr (DUAL) {
        const int lo = (int)((int64_t)j.w.kf * ks / A.ksplit), hi = (int)((int64_t)j.w.kf * (ks + 1) / A.ksplit);
        if (lo < j.kf1) {
            run(j.x, lo, min(hi, j.kf1), 0);
            store(j.scale1, true);
            clear();
        }
        if (hi > j.kf1) {
            run(j.x2, max(lo, j.kf1), hi, j.kf1);
            store(j.scale2, lo >= j.kf1);
        }
    } else {
        run(j.x, 0, j.w.kf, 0);
        store(nullptr, true);
    }
}

template <int KA, int RT, int CT> void launch_lds_groups(hipStream_t s, DenseArgs & A) {
    A.n_groups = (A.j.w.tiles + 2 * RT - 1) / (2 * RT);
    const int tiles = (A.groups.max_tiles + 7) / 8 * 8;
    hipLaunchKernelGGL((k_dense_lds<KA, -1, RT, CT, true>), dim3((unsigned)(A.n_groups * tiles)), dim3(256), 0, s, A, tiles);
}
template <typename TA, int KA, int RT, int CT, int KW, int RW> void launch_groups(hipStream_t s, DenseArgs & A) {
    A.n_groups = (A.j.w.tiles + RT * RW - 1) / (RT * RW);
    const dim3 grid((unsigned)A.n_groups, (unsigned)A.groups.max_tiles);
    hipLaunchKernelGGL((k_dense<TA, KA, -1, RT, CT, KW, RW, true>), grid, dim3(64 * KW * RW), 0, s, A);
}

template <int KA, int KB, int RT, int CT> void launch_lds(hipStream_t s, DenseArgs & A) {
    A.n_groups = (A.j.w.tiles + 2 * RT - 1) / (2 * RT);
    const int tok_blocks = (A.T + 32 * CT - 1) / (32 * CT), bands = (tok_blocks + 7) / 8;
    A.grid_k = 8 * bands * 8 * ((A.n_groups + 7) / 8);
    hipLaunchKernelGGL((k_dense_lds<KA, KB, RT, CT, false>), dim3((unsigned)(A.grid_k * A.ksplit)), dim3(256), 0, s, A, tok_blocks);
}

template <typename TA, int KA, int KB, int RT, int CT, int KW, int RW> void launch(hipStream_t s, DenseArgs & A) {
    const DenseJob & j = A.j;
    A.n_groups = (j.w.tiles + RT * RW - 1) / (RT * RW);
    const dim3 grid((unsigned)(A.n_groups * A.ksplit), (unsigned)((A.T + 16 * CT - 1) / (16 * CT)), (unsigned)j.w.batch);
    hipLaunchKernelGGL((k_dense<TA, KA, KB, RT, CT, KW, RW, false>), grid, dim3(64 * KW * RW), 0, s, A);
}

constexpr int kMaxSlices = 8;
constexpr size_t kSliceFloats = (size_t)64 * 32768;      // tokens x rows of one slice

template <int KA, int KB> Slices run(hipStream_t s, int arith, DenseArgs & A, float * ws) {
    Slices out;
    const int T = A.T;
    const DenseWeight & w = A.j.w;
    constexpr bool PAIRS = out_is_glu(KA) || out_is_glu(KB);      // row tiles in pairs
    constexpr int R1 = PAIRS ? 2 : 1;
    auto slices = [&](int n) {
        A.ksplit = n;
        A.partial = ws;
        A.slice = (size_t)T * w.n;
        out.data = ws;
        out.n = n;
        out.stride = A.slice;
        out.N = w.n;
    };
    if (KA == OUT_RESIDUAL && !A.j.a.dst) slices(1);
    if (arith == ARITH_32) {
        if (T <= 16) launch<float, KA, KB, R1, 1, 4, 1>(s, A);
        else launch<float, KA, KB, 2, 4, 1, 4>(s, A);
        return out;
    }
    // K-slices: workgroups that share rows along K leave partial results, added by the next norm
    auto slice_k = [&](int want, int least) {            // least: fragments of a slice
        const int n = std::min({kMaxSlices, want, w.kf / least});
        if (n > 1) slices(n);
    };
    const bool sliceable = KA == OUT_RESIDUAL && ws && (size_t)T * w.n <= kSliceFloats;
    if constexpr (KA != OUT_QUERY && KA != OUT_ACT_GATED) {        // products of one matrix
        auto blocks = [&](int rt, int ct) { return (int64_t)((w.tiles + 2 * rt - 1) / (2 * rt)) * ((T + 32 * ct - 1) / (32 * ct)); };
        if (w.batch == 1 && T > 128) {
            // the largest tile that leaves every CU a workgroup
            if constexpr (KA != OUT_RESIDUAL) {
                if (blocks(8, 4) >= 448) { launch_lds<KA, KB, 8, 4>(s, A); return out; }
            }
            if (sliceable && w.n % 4 == 0 && blocks(4, 4) < 256) {
                slice_k((int)(512 / blocks(4, 4)), 16);
                launch_lds<KA, KB, 4, 4>(s, A);
            } else if (blocks(4, 4) >= 256) launch_lds<KA, KB, 4, 4>(s, A);
            else launch_lds<KA, KB, 4, 2>(s, A);
            return out;
        }
    }
    const bool deep = w.kf >= 16;
    if (deep && sliceable) slice_k(512 / std::max(T <= 16 ? w.tiles : (w.tiles + 1) / 2, 1), 64);
    if (!deep) {                        // one wave has too little of K to share it
        if (T <= 16) launch<uint16_t, KA, KB, R1, 1, 1, 4>(s, A);
        else if (T <= 32) launch<uint16_t, KA, KB, R1, 2, 1, 4>(s, A);
        else launch<uint16_t, KA, KB, R1, 4, 1, 4>(s, A);
    } else if (T <= 16) launch<uint16_t, KA, KB, R1, 1, 8, 1>(s, A);
    else if (T <= 32) launch<uint16_t, KA, KB, 2, 2, 8, 1>(s, A);
    else if (!PAIRS && (int64_t)w.tiles * A.ksplit * w.batch <= 256) launch<uint16_t, KA, KB, R1, 4, 8, 1>(s, A);      // a workgroup for every row tile
    else launch<uint16_t, KA, KB, 2, 4, 8, 1>(s, A);
    return out;
}

// Products of the pairs of every expert: short tiles straight to registers, longer ones through LDS.
template <int KA> void run_groups(hipStream_t s, int arith, DenseArgs & A) {
    constexpr int R1 = out_is_glu(KA) ? 2 : 1;
    const int block = A.groups.block;
    if (arith == ARITH_32) {
        if (block == 16) launch_groups<float, KA, R1, 1, 4, 1>(s, A);
        else launch_groups<float, KA, 2, 4, 1, 4>(s, A);
        return;
    }
    const bool deep = A.j.w.kf >= 16;
    switch (block) {
        case 16: deep ? launch_groups<uint16_t, KA, R1, 1, 8, 1>(s, A) : launch_groups<uint16_t, KA, R1, 1, 1, 4>(s, A); break;
        case 32: deep ? launch_groups<uint16_t, KA, 2, 2, 8, 1>(s, A) : launch_groups<uint16_t, KA, R1, 2, 1, 4>(s, A); break;
        case 64: launch_lds_groups<KA, 4, 2>(s, A); break;
        default:
            if (out_is_glu(KA) && (int64_t)A.groups.max_tiles * ((A.j.w.tiles + 15) / 16) >= 448) launch_lds_groups<KA, 8, 4>(s, A);
            else launch_lds_groups<KA, 4, 4>(s, A);
            break;
    }
}

}  // namespace

int expert_block(int arith, int T, int top, int experts) {
    const int mean = (T * top + experts - 1) / experts;      // pairs of an expert
    if (arith == ARITH_32) return mean <= 16 ? 16 : 64;
    return mean <= 8 ? 16 : mean <= 24 ? 32 : mean <= 96 ? 64 : 128;
}

void dense_pack(hipStream_t s, const uint16_t * src, int rows, int cols, int64_t row_stride, int64_t k_stride,
                uint16_t * dst, int kf, PackMap row, PackMap column) {
    if (rows <= 0 || cols <= 0) return;
    const int64_t n = (int64_t)rows * cols;
    hipLaunchKernelGGL(k_dense_pack, dim3((unsigned)std::min<int64_t>((n + 255) / 256, 8192)), dim3(256), 0, s, src, rows, cols,
                       row_stride, k_stride, dst, kf, row, column);
    check_launch("dense_pack");
}

size_t dense_workspace_floats() { return kMaxSlices * kSliceFloats; }

Slices dense(hipStream_t s, int arith, const DenseJob & job, int T, float * ws) {
    if (T <= 0 || job.w.n <= 0) return Slices();
    DenseArgs A;
    A.j = job;
    A.T = T;
    A.ksplit = 1;
    A.partial = nullptr;
    A.slice = 0;
    if (job.groups) {
        A.groups = *job.groups;
        if (A.groups.max_tiles <= 0) return Slices();
        A.j.split_tile = A.j.w.tiles;
        A.j.n_a = A.j.w.n;
        switch (job.a.kind) {
            case OUT_ACT_SWIGLU: run_groups<OUT_ACT_SWIGLU>(s, arith, A); break;
            case OUT_ACT_CLAMPED: run_groups<OUT_ACT_CLAMPED>(s, arith, A); break;
            case OUT_EXPERT: run_groups<OUT_EXPERT>(s, arith, A); break;
            default: throw std::runtime_error("dense: this output of an expert product is not compiled");
        }
        check_launch("dense");
        return Slices();
    }
    const bool two = A.j.n_a > 0 && A.j.split_tile < A.j.w.tiles;
    if (!two) { A.j.split_tile = A.j.w.tiles; A.j.n_a = A.j.w.n; }
    Slices out;
    if (two) {
        if (job.a.kind == OUT_F32 && job.b.kind == OUT_ACT_RELU2) out = run<OUT_F32, OUT_ACT_RELU2>(s, arith, A, ws);
        else if (job.a.kind == OUT_F32 && job.b.kind == OUT_ACT_SWIGLU) out = run<OUT_F32, OUT_ACT_SWIGLU>(s, arith, A, ws);
        else if (job.a.kind == OUT_F32 && job.b.kind == OUT_ACT_CLAMPED) out = run<OUT_F32, OUT_ACT_CLAMPED>(s, arith, A, ws);
        else if (job.a.kind == OUT_F32 && job.b.kind == OUT_ACT) out = run<OUT_F32, OUT_ACT>(s, arith, A, ws);
        else if (job.a.kind == OUT_ROTARY && job.b.kind == OUT_F32) out = run<OUT_ROTARY, OUT_F32>(s, arith, A, ws);
        else throw std::runtime_error("dense: this pair of outputs is not compiled");
    } else {
        switch (job.a.kind) {
            case OUT_F32: out = run<OUT_F32, -1>(s, arith, A, ws); break;
            case OUT_ACT: out = run<OUT_ACT, -1>(s, arith, A, ws); break;
            case OUT_ACT_GATED: out = run<OUT_ACT_GATED, -1>(s, arith, A, ws); break;
            case OUT_ACT_GEGLU: out = run<OUT_ACT_GEGLU, -1>(s, arith, A, ws); break;
            case OUT_ACT_SWIGLU: out = run<OUT_ACT_SWIGLU, -1>(s, arith, A, ws); break;
            case OUT_ACT_CLAMPED: out = run<OUT_ACT_CLAMPED, -1>(s, arith, A, ws); break;
            case OUT_F32_CAPPED: out = run<OUT_F32_CAPPED, -1>(s, arith, A, ws); break;
            case OUT_ACT_RELU2: out = run<OUT_ACT_RELU2, -1>(s, arith, A, ws); break;
            case OUT_ROTARY: out = run<OUT_ROTARY, -1>(s, arith, A, ws); break;
            case OUT_QUERY: out = run<OUT_QUERY, -1>(s, arith, A, ws); break;
            case OUT_RESIDUAL: out = run<OUT_RESIDUAL, -1>(s, arith, A, ws); break;
            default: throw std::runtime_error("dense: this output is not compiled");
        }
    }
    check_launch("dense");
    return out;
}

}  // namespace rk
