// Paged attention of layer-stack models, in two forms that share their kernels.
// Latent: keys and values of every head are up-projections of one cached latent per token, so a query is absorbed into
// the latent space first (q' = W_uk^T q) and every head attends over the same cached rows, which are keys and values at
// once. The attended latents leave as activations for the value up-projection.
// Grouped: a cache of keys and one of values, each with a part per key/value head, of one width or of two, and optionally
// soft-capped scores.
// Either sees all earlier positions, a sliding window of them, or those of the token's own chunk.
#include "stack_dev.hpp"

namespace rk {

namespace {

template <typename EL> __device__ __forceinline__ float el_float(EL v);
template <> __device__ __forceinline__ float el_float<__half>(__half v) { return __half2float(v); }
template <> __device__ __forceinline__ float el_float<float>(float v) { return v; }
template <typename EL> __device__ __forceinline__ EL float_el(float v);
template <> __device__ __forceinline__ __half float_el<__half>(float v) { return sat_half(v); }
template <> __device__ __forceinline__ float float_el<float>(float v) { return v; }

// One workgroup per token and norm: the queries' latent, and (blockIdx.y = 1) the latent that goes into the cache. A
// thread keeps its groups of eight columns in registers between the two passes.
template <int ARITH>
__global__ __launch_bounds__(256) void k_latent_norms(LatentNorms a) {
    using EL = typename std::conditional<ARITH == ARITH_16, __half, float>::type;
    __shared__ float scratch[16];
    constexpr int KEEP = 2;                    // groups of eight per thread that stay in registers
    const int t = blockIdx.x;
    const bool kv = blockIdx.y == 1;
    const int n = kv ? a.kv_rank : a.q_rank;
    const float * src = a.proj + (size_t)t * a.ld + (kv ? a.kv_col : 0);
    const float * w = kv ? a.kv_w : a.q_w;
    float v[KEEP][8], q = 0.0f;
    auto load = [&](int k, float (&o)[8]) {    // rows of the product start at multiples of four
        if (k + 8 <= n) {
            const f4 x = *(const f4 *)(src + k), y = *(const f4 *)(src + k + 4);
#pragma unroll
            for (int i = 0; i < 4; ++i) { o[i] = x[i]; o[4 + i] = y[i]; }
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) o[i] = k + i < n ? src[k + i] : 0.0f;
        }
    };
#pragma unroll
    for (int g = 0; g < KEEP; ++g) {
        load(8 * (int)(threadIdx.x + 256 * g), v[g]);
#pragma unroll
        for (int i = 0; i < 8; ++i) q += v[g][i] * v[g][i];
    }
    for (int k = 8 * (int)(threadIdx.x + 256 * KEEP); k < n; k += 8 * 256) {
        float o[8];
        load(k, o);
#pragma unroll
        for (int i = 0; i < 8; ++i) q += o[i] * o[i];
    }
    q = block_sum(q, scratch);
    const float inv = 1.0f / sqrtf(q / (float)n + a.eps);
    const int cell = kv ? a.cell[t] : 0;
    EL * page = kv ? (EL *)a.pool + (size_t)(cell / PAGE) * cache_page_elems(a.pool_kf) : nullptr;
    const int padded = 32 * (kv ? a.pool_kf : a.act_q_kf);
    auto finish = [&](int k, float (&o)[8]) {
        if (k >= padded) return;
#pragma unroll
        for (int i = 0; i < 8; ++i) o[i] = k + i < n ? o[i] * inv * w[k + i] : 0.0f;
        if (kv) {
            EL * dst = page + cache_at(cell % PAGE, k);
#pragma unroll
            for (int i = 0; i < 8; ++i) dst[i] = float_el<EL>(o[i]);
        } else {
            store_frag8<ARITH>(a.act_q, a.act_q_kf, t, k, o);
        }
    };
#pragma unroll
    for (int g = 0; g < KEEP; ++g) finish(8 * (int)(threadIdx.x + 256 * g), v[g]);
    for (int k = 8 * (int)(threadIdx.x + 256 * KEEP); k < padded; k += 8 * 256) {
        float o[8];
        load(k, o);
        finish(k, o);
    }
}

template <int ARITH, typename EL> __device__ __forceinline__ void store_el8(EL * dst, const float (&v)[8]) {
    if constexpr (ARITH == ARITH_16) {
        union { __half h[8]; u4 w; } p;
#pragma unroll
        for (int i = 0; i < 8; ++i) p.h[i] = sat_half(v[i]);
        *(u4 *)dst = p.w;
    } else {
        *(f4 *)dst = f4{v[0], v[1], v[2], v[3]};
        *(f4 *)(dst + 4) = f4{v[4], v[5], v[6], v[7]};
    }
}

// One workgroup per token: the squares of all queries and all keys, then every head in groups of eight columns.
template <int ARITH>
__global__ __launch_bounds__(256) void k_head_rows(HeadRows a) {
    using EL = typename std::conditional<ARITH == ARITH_16, __half, float>::type;
    __shared__ float scratch[16];
    const int t = blockIdx.x;
    const float * row = a.proj + (size_t)t * a.ld;
    auto squares = [&](const float * x, int n) {       // rows start at multiples of four columns
        float q = 0.0f;
        const int whole = n / 4 * 4;
        for (int k = 4 * (int)threadIdx.x; k < whole; k += 1024) {
            const f4 v = *(const f4 *)(x + k);
            q += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
        for (int k = whole + (int)threadIdx.x; k < n; k += 256) q += x[k] * x[k];
        return 1.0f / sqrtf(block_sum(q, scratch) / (float)n + a.eps);
    };
    const float inv_q = squares(row + a.q_col, a.H * a.dim), inv_k = squares(row + a.k_col, a.G * a.dim);
    auto load = [](const float * x, int n, bool aligned, float (&o)[8]) {      // n columns are left
        if (aligned && n >= 8) {
            const f4 u = *(const f4 *)x, v = *(const f4 *)(x + 4);
#pragma unroll
            for (int i = 0; i < 4; ++i) { o[i] = u[i]; o[4 + i] = v[i]; }
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) o[i] = i < n ? x[i] : 0.0f;
        }
    };
    const int per_k = a.kf * 4, per_v = a.vf * 4;       // groups of a head
    const bool even = a.dim % 4 == 0, even_v = a.vdim % 4 == 0;
    const int cell = a.cell[t];
    EL * k_page = (EL *)a.k_pool + (size_t)(cell / PAGE) * cache_page_elems(a.kf * a.G);
    EL * v_page = (EL *)a.v_pool + (size_t)(cell / PAGE) * cache_page_elems(a.vf * a.G);
    for (int i = threadIdx.x; i < (a.H + a.G) * per_k; i += 256) {
        const int head = i / per_k, c = (i - head * per_k) * 8;
        const bool query = head < a.H;
        const int h = query ? head : head - a.H, left = a.dim - c;
        float v[8], w[8];
        load(row + (query ? a.q_col : a.k_col) + h * a.dim + c, left, even, v);
        load((query ? a.q_w : a.k_w) + h * a.dim + c, left, even, w);
        const float inv = query ? inv_q : inv_k;
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = v[e] * inv * w[e];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int pair = c / 2 + e;
            if (pair >= a.pairs) continue;
            const float2 cs = *(const float2 *)(a.table + 2 * ((size_t)t * a.pairs + pair));
            const float x = v[2 * e], y = v[2 * e + 1];
            v[2 * e] = x * cs.x - y * cs.y;
            v[2 * e + 1] = y * cs.x + x * cs.y;
        }
        if (query) store_el8<ARITH>((EL *)a.q + ((size_t)t * a.H + h) * (a.kf * 32) + c, v);
        else store_el8<ARITH>(k_page + cache_at(cell % PAGE, h * a.kf * 32 + c), v);
    }
    const float share = a.share ? *a.share : 0.0f;
    for (int i = threadIdx.x; i < a.G * per_v; i += 256) {
        const int h = i / per_v, c = (i - h * per_v) * 8, left = a.vdim - c;
        float v[8];
        load(row + a.v_col + h * a.vdim + c, left, even_v, v);
        if (a.first) {
            float * f = a.first + (size_t)t * a.G * a.vdim + h * a.vdim + c;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                if (e >= left) break;
                if (a.share) v[e] = (1.0f - share) * v[e] + share * f[e];
                else f[e] = v[e];
            }
        }
        store_el8<ARITH>(v_page + cache_at(cell % PAGE, h * a.vf * 32 + c), v);
    }
}

// First position a token at `pos` sees.
__device__ __forceinline__ int low_key(const StackAttn & a, int kv_begin, int pos) {
    return max(kv_begin, a.chunk > 0 ? pos - pos % a.chunk : a.window > 0 ? pos - a.window + 1 : 0);
}

// Any width, either element type: one workgroup per query column, keys in batches of one per thread, f32 throughout.
template <int ARITH>
__global__ __launch_bounds__(256) void k_stack_attention_any(StackAttn a) {
    using EL = typename std::conditional<ARITH == ARITH_16, __half, float>::type;
    extern __shared__ float sm[];
    const int R = a.kf * 32, V = a.vf * 32, HG = a.H / a.G, kv_head = blockIdx.y;
    float * q = sm, * p = sm + R;             // [R], [256]
    __shared__ float scratch[16];
    const AttnBlock blk = a.blocks[blockIdx.x];
    const RowDesc row = a.rows[blk.row];
    const int n_cols = row.n * HG;
    const size_t page_elems = cache_page_elems(a.kf * a.G), v_page_elems = cache_page_elems(a.vf * a.G);
    const EL * keys = (const EL *)a.pool + cache_page_elems(a.kf * kv_head);
    const EL * values = (const EL *)(a.v_pool ? a.v_pool : a.pool) + cache_page_elems(a.vf * kv_head);
    constexpr float LOG2E = 1.4426950408889634f;
    for (int c = blk.col0; c < min(blk.col0 + a.block_cols, n_cols); ++c) {
        const int tok = c / HG, h = kv_head * HG + c % HG, t = row.tok_off + tok, pos = row.pos0 + tok;
        const int lo = low_key(a, row.kv_begin, pos);
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
                const EL * page = keys + (size_t)pg * page_elems;
                s = 0.0f;
                for (int k = 0; k < R; k += 8) {
                    const EL * e = page + cache_at(key % PAGE, k);
#pragma unroll
                    for (int i = 0; i < 8; ++i) s += q[k + i] * el_float<EL>(e[i]);
                }
                if (a.v_pool) {
                    s *= a.scale;
                    if (a.softcap > 0.0f) s = a.softcap * tanhf(s / a.softcap);
                    s *= LOG2E;
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
                const EL * page = values + (size_t)pg * v_page_elems;
                const float pk = p[k];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int col = threadIdx.x + 256 * i;
                    if (col < V) acc[i] += pk * el_float<EL>(page[cache_at(kk % PAGE, col)]);
                }
            }
        }
        const float inv = 1.0f / l;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int col = threadIdx.x + 256 * i;
            if (col >= V) break;
            const size_t at = frag_at(t, h * V + col, a.out_kf);
            if constexpr (ARITH == ARITH_16) ((uint16_t *)a.out)[at] = bf16_bits(acc[i] * inv);
            else ((float *)a.out)[at] = acc[i] * inv;
        }
    }
}

typedef __fp16 q4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) q4 lds_q4;

// Matrix-core form over f16 cache rows of KF fragments (per head; values of VF). A workgroup serves CT * WC * 16 query columns of one
// key/value head (blockIdx.z); WC waves share a page (staged once into LDS, double buffered, by direct-to-LDS loads), WK
// such groups take pages in turn and merge at the end. Scores S^T = K q^T and outputs O^T = V^T P^T read pages of one
// layout: the second product's operand is its transpose, which the LDS transpose read delivers, so rows that are keys
// and values at once (KV false) are staged once; KV: a page of keys, then the page of values. With several splits
// (blockIdx.y) every one leaves an unnormalised partial result.
template <int KF, int VF, int CT, int WC, int WK, bool KV>
__global__ __launch_bounds__(64 * WC * WK) __attribute__((amdgpu_waves_per_eu(2, 2)))
void k_stack_attention(StackAttn a) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    __shared__ float merge_ml[WC][CT][2][64];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int wc = wave % WC, wk = wave / WC, g = lane >> 4;
    static_assert(KV || KF == VF);
    constexpr int AHEAD = KF >= 4 ? 6 : 2 * KF, AHEAD_V = VF >= 4 ? 6 : 2 * VF;
    constexpr int kf = KF, head_bytes = KF * 2048, value_bytes = VF * 2048, page_bytes = head_bytes + (KV ? value_bytes : 0);      // of a staged page
    constexpr int PIECES = page_bytes / 1024;
    const AttnBlock blk = a.blocks[blockIdx.x];
    const RowDesc row = a.rows[blk.row];
    const int HG = KV ? a.H / a.G : a.H, kv_head = KV ? blockIdx.z : 0;
    const int n_cols = row.n * HG;
    auto low_of = [&](int pos) { return low_key(a, row.kv_begin, pos); };

    // the block's pages, dealt to the splits
    const int last_tok = min(blk.col0 + a.block_cols, n_cols) - 1;
    const int page_lo = low_of(row.pos0 + blk.col0 / HG) / PAGE, page_hi = (row.pos0 + last_tok / HG) / PAGE + 1;
    const int n_all = page_hi - page_lo, sp = blockIdx.y;
    const int first = page_lo + (int)((int64_t)n_all * sp / a.splits), end = page_lo + (int)((int64_t)n_all * (sp + 1) / a.splits);
    const int n_iter = (end - first + WK - 1) / WK;
    const int32_t * table = a.table + (size_t)row.slot * a.max_pages;
    uint8_t * buf = lds + (size_t)wk * 2 * page_bytes;
    const uint32_t to = lds_offset(lds) + (uint32_t)(wk * 2 * page_bytes);

    auto stage = [&](int page, int b) {
        if (page >= end) return;
        // a scalar load, which no vector load is waited for with
        const int id = __builtin_amdgcn_readfirstlane(((const __attribute__((address_space(4))) int32_t *)table)[__builtin_amdgcn_readfirstlane(page)]);
        const size_t at = KV ? ((size_t)id * a.G + kv_head) * head_bytes : (size_t)id * head_bytes;
        const uint8_t * src = (const uint8_t *)a.pool + at;
        const uint8_t * src_v = KV ? (const uint8_t *)a.v_pool + ((size_t)id * a.G + kv_head) * value_bytes - head_bytes : src;
        for (int ch = wc; ch < PIECES; ch += WC)
            lds_dma16((ch < 2 * kf ? src : src_v) + ch * 1024, (uint32_t)lane * 16, __builtin_amdgcn_readfirstlane(to + (uint32_t)(b * page_bytes + ch * 1024)));
    };
    // this lane's column of every column tile: its token and head, and the keys it sees
    int col[CT], lo[CT], hi[CT], lo_max = 0, hi_min = 1 << 30;
    h8 q[CT][KF];
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        col[c] = blk.col0 + (wc * CT + c) * 16 + (lane & 15);
        const int cc = min(col[c], n_cols - 1);
        const int tok = cc / HG, h = kv_head * HG + cc - tok * HG;
        hi[c] = row.pos0 + tok;
        lo[c] = low_of(hi[c]);
        lo_max = max(lo_max, lo[c]);
        hi_min = min(hi_min, hi[c]);
        const __half * qr = (const __half *)a.q + ((size_t)(row.tok_off + tok) * a.H + h) * (size_t)(kf * 32) + 8 * g;
#pragma unroll
        for (int j = 0; j < KF; ++j) q[c][j] = load_h8(qr + 32 * j);
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) {
        lo_max = max(lo_max, __shfl_xor(lo_max, o, 64));
        hi_min = min(hi_min, __shfl_xor(hi_min, o, 64));
    }
    constexpr float LOG2E = 1.4426950408889634f;
    const float cap_out = KV ? a.softcap * LOG2E : 0.0f;
    const float score_in = KV ? (a.softcap > 0.0f ? 2.0f * LOG2E * a.scale / a.softcap : a.scale * LOG2E) : 1.0f;
    f4 acc[CT][2 * VF];
    float m[CT], l[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        m[c] = -INFINITY;
        l[c] = 0.0f;
#pragma unroll
        for (int d = 0; d < 2 * VF; ++d) acc[c][d] = f4{0, 0, 0, 0};
    }
    const int idx = lane & 15;
    const int tr_lane = ((((idx >> 1) & 1) * 16 + 4 * g + (idx >> 2)) * 8 + (idx & 1) * 4) * 2;       // bytes into a 1 KiB piece
    stage(first + wk, 0);
    stage(first + wk + WK, 1);
#pragma unroll
    for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int j = 0; j < KF; ++j) asm volatile("" :: "v"(q[c][j]));      // the queries are waited for here, not in the loop
    for (int it = 0; it < n_iter; ++it) {
        // a page's loads and the next one's are on their way: wait for the former
        const int page = first + it * WK + wk;
        if (it > 0) {
            __syncthreads();
            stage(page + WK, (it + 1) & 1);
        }
        if (page + WK < end) asm volatile("s_waitcnt vmcnt(%0)" :: "n"(PIECES / WC) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (page >= end) continue;
        const uint8_t * cur = buf + (size_t)(it & 1) * page_bytes;
        f4 s[2][CT];
#pragma unroll
        for (int hf = 0; hf < 2; ++hf) {
#pragma unroll
            for (int c = 0; c < CT; ++c) s[hf][c] = f4{0, 0, 0, 0};
#pragma unroll
            for (int j = 0; j < KF; ++j) {
                const h8 k = *(const h8 *)(cur + (j * 2 + hf) * 1024 + lane * 16);
#pragma unroll
                for (int c = 0; c < CT; ++c) s[hf][c] = __builtin_amdgcn_mfma_f32_16x16x32_f16(k, q[c][j], s[hf][c], 0, 0, 0);
            }
        }
        // eight reads ahead of the products: the scheduler would otherwise wait for every read it issues
        __builtin_amdgcn_sched_group_barrier(0x100, AHEAD, 0);
#pragma unroll
        for (int i = 0; i < 2 * KF - AHEAD; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x008, CT, 0);
            __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        }
        __builtin_amdgcn_sched_group_barrier(0x008, AHEAD * CT, 0);
        if constexpr (KV) {       // scores in powers of two; tanh(x) = 1 - 2 / (1 + e^2x)
            if (cap_out > 0.0f) {
#pragma unroll
                for (int hf = 0; hf < 2; ++hf)
#pragma unroll
                    for (int c = 0; c < CT; ++c)
#pragma unroll
                        for (int i = 0; i < 4; ++i) {
                            const float e = __builtin_amdgcn_exp2f(s[hf][c][i] * score_in);
                            s[hf][c][i] = fmaf(-2.0f * cap_out, __builtin_amdgcn_rcpf(1.0f + e), cap_out);
                        }
            } else {
#pragma unroll
                for (int hf = 0; hf < 2; ++hf)
#pragma unroll
                    for (int c = 0; c < CT; ++c) s[hf][c] *= score_in;
            }
        }
        const int key0 = page * PAGE;
        const bool inside = key0 >= lo_max && key0 + PAGE - 1 <= hi_min;
        h8 p[CT];
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            if (!inside) {
#pragma unroll
                for (int hf = 0; hf < 2; ++hf)
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const int key = key0 + hf * 16 + 4 * g + i;
                        if (key < lo[c] || key > hi[c]) s[hf][c][i] = -INFINITY;
                    }
            }
            float mx = fmaxf(fmaxf(fmaxf(s[0][c][0], s[0][c][1]), fmaxf(s[0][c][2], s[0][c][3])),
                             fmaxf(fmaxf(s[1][c][0], s[1][c][1]), fmaxf(s[1][c][2], s[1][c][3])));
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            const float m2 = fmaxf(m[c], mx), base = m2 == -INFINITY ? 0.0f : m2;
            if (__ballot(m2 > m[c])) {
                const float f = exp2f(m[c] - base);
                l[c] *= f;
#pragma unroll
                for (int d = 0; d < 2 * VF; ++d) acc[c][d] *= f;
                m[c] = m2;
            }
#pragma unroll
            for (int hf = 0; hf < 2; ++hf)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float e = exp2f(s[hf][c][i] - base);
                    l[c] += e;
                    p[c][hf * 4 + i] = (_Float16)e;
                }
        }
#pragma unroll
        for (int d = 0; d < 2 * VF; ++d) {
            const uint8_t * v0 = cur + (KV ? head_bytes : 0) + (d >> 1) * 2048 + (d & 1) * 512 + tr_lane;
            union { q4 half[2]; h8 all; } v;
            v.half[0] = __builtin_amdgcn_ds_read_tr16_b64_v4f16((lds_q4 *)(v0));
            v.half[1] = __builtin_amdgcn_ds_read_tr16_b64_v4f16((lds_q4 *)(v0 + 1024));
#pragma unroll
            for (int c = 0; c < CT; ++c) acc[c][d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v.all, p[c], acc[c][d], 0, 0, 0);
        }
        __builtin_amdgcn_sched_group_barrier(0x100, 2 * AHEAD_V, 1);
#pragma unroll
        for (int i = 0; i < 2 * VF - AHEAD_V; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x008, CT, 1);
            __builtin_amdgcn_sched_group_barrier(0x100, 2, 1);
        }
        __builtin_amdgcn_sched_group_barrier(0x008, AHEAD_V * CT, 1);
    }
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        l[c] += __shfl_xor(l[c], 16, 64);
        l[c] += __shfl_xor(l[c], 32, 64);
    }
    if constexpr (WK > 1) {       // the groups' results, one after the other, into the first group's
        static_assert(WK == 2 && CT == 1);
        __syncthreads();
        f4 * park = (f4 *)lds + (size_t)wc * 2 * VF * 64;      // 2 KiB per fragment and wave: within the pages
        if (wk == 1) {
            merge_ml[wc][0][0][lane] = m[0];
            merge_ml[wc][0][1][lane] = l[0];
#pragma unroll
            for (int d = 0; d < 2 * VF; ++d) park[d * 64 + lane] = acc[0][d];
        }
        __syncthreads();
        if (wk == 1) return;
        const float mo = merge_ml[wc][0][0][lane], lo2 = merge_ml[wc][0][1][lane];
        const float m2 = fmaxf(m[0], mo), base = m2 == -INFINITY ? 0.0f : m2;
        const float f0 = exp2f(m[0] - base), f1 = exp2f(mo - base);
        l[0] = l[0] * f0 + lo2 * f1;
        m[0] = m2;
#pragma unroll
        for (int d = 0; d < 2 * VF; ++d) acc[0][d] = acc[0][d] * f0 + park[d * 64 + lane] * f1;
    }
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        if (col[c] >= min(blk.col0 + a.block_cols, n_cols)) continue;
        const int tok = col[c] / HG, h = kv_head * HG + col[c] - tok * HG, t = row.tok_off + tok;
        if (a.splits > 1) {
            const size_t at = ((size_t)t * a.H + h) * a.splits + sp;
            if (g == 0) *(float2 *)(a.partial_ml + 2 * at) = make_float2(m[c], l[c]);
            __half * o = (__half *)a.partial + at * (size_t)(VF * 32);
            const float inv = l[c] > 0.0f ? 1.0f / l[c] : 0.0f;      // a split may lie outside this column's window
#pragma unroll
            for (int d = 0; d < 2 * VF; ++d) {
                union { __half h[4]; uint2 u; } w;
#pragma unroll
                for (int i = 0; i < 4; ++i) w.h[i] = __float2half_rn(acc[c][d][i] * inv);
                *(uint2 *)(o + d * 16 + 4 * g) = w.u;
            }
        } else {
            const float inv = 1.0f / l[c];
#pragma unroll
            for (int d = 0; d < 2 * VF; ++d) {
                const f4 v = acc[c][d] * inv;
                uint2 u;
                u.x = (uint32_t)bf16_bits(v[0]) | ((uint32_t)bf16_bits(v[1]) << 16);
                u.y = (uint32_t)bf16_bits(v[2]) | ((uint32_t)bf16_bits(v[3]) << 16);
                *(uint2 *)((uint16_t *)a.out + frag_at(t, h * VF * 32 + d * 16 + 4 * g, a.out_kf)) = u;
            }
        }
    }
}

// Merges the splits of one query column (at most 32), each a mean in f16 with its maximum and sum: a wave per column,
// lane i the weight of split i; eight latent columns per lane and pass, the splits' values requested four at a time.
__global__ __launch_bounds__(64) void k_stack_combine(StackAttn a) {
    const int R = a.vf * 32, t = blockIdx.x / a.H, h = blockIdx.x - t * a.H, lane = threadIdx.x;
    const __half * p = (const __half *)a.partial + (size_t)blockIdx.x * a.splits * R;
    const float * ml = a.partial_ml + (size_t)blockIdx.x * a.splits * 2;
    const float m = lane < a.splits ? ml[2 * lane] : -INFINITY, l = lane < a.splits ? ml[2 * lane + 1] : 0.0f;
    float top = m;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) top = fmaxf(top, __shfl_xor(top, o, 64));
    const float f = l * exp2f(m - top);
    const float mine = f / wave_sum(f);
    for (int k0 = 0; k0 < R; k0 += 512) {
        const int k = k0 + 8 * lane, kc = min(k, R - 8);
        float v[8] = {};
        for (int s = 0; s < a.splits; s += 4) {
            h8 u[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) u[i] = load_h8(p + (size_t)min(s + i, a.splits - 1) * R + kc);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float c = s + i < a.splits ? __shfl(mine, s + i, 64) : 0.0f;
#pragma unroll
                for (int e = 0; e < 8; ++e) v[e] += (float)u[i][e] * c;
            }
        }
        if (k < R) store_frag8<ARITH_16>(a.out, a.out_kf, t, h * R + k, v);
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
__global__ void k_stack_cells(EL * __restrict__ pool, int kf, const int32_t * __restrict__ cells, int n, EL * __restrict__ rows, bool gather) {
    const int groups = kf * 4;
    const int64_t total = (int64_t)n * groups;
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (int64_t)gridDim.x * blockDim.x) {
        const int r = (int)(i / groups), c = (int)(i % groups) * 8;
        const int cell = cells[r];
        EL * p = pool + (size_t)(cell / PAGE) * cache_page_elems(kf) + cache_at(cell % PAGE, c);
        EL * o = rows + (size_t)r * kf * 32 + c;
#pragma unroll
        for (int k = 0; k < 8; ++k) { if (gather) o[k] = p[k]; else p[k] = o[k]; }
    }
}

}  // namespace

void latent_norms(hipStream_t s, int arith, const LatentNorms & a, int T) {
    if (T <= 0) return;
    const dim3 grid((unsigned)T, a.kv_w ? 2u : 1u);
    if (arith == ARITH_16) hipLaunchKernelGGL(k_latent_norms<ARITH_16>, grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL(k_latent_norms<ARITH_32>, grid, dim3(256), 0, s, a);
    check_launch("latent_norms");
}

void head_rows(hipStream_t s, int arith, const HeadRows & a, int T) {
    if (T <= 0) return;
    if (arith == ARITH_16) hipLaunchKernelGGL(k_head_rows<ARITH_16>, dim3((unsigned)T), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(k_head_rows<ARITH_32>, dim3((unsigned)T), dim3(256), 0, s, a);
    check_launch("head_rows");
}

namespace {
// Widest cache rows (in fragments) of the matrix-core kernel: rows that are keys and values at once, and separate ones.
constexpr int kMatrixKf = 16, kMatrixKfPair = 8;
// Widths of keys and values where they differ.
constexpr PairFrags kPairs[] = {{3, 1}, {4, 2}, {2, 4}, {6, 4}, {8, 4}, {4, 8}};
bool on_matrix_cores(int arith, int kf, int vf, bool pair) { return arith == ARITH_16 && std::max(kf, vf) <= (pair ? kMatrixKfPair : kMatrixKf); }

template <int KF, int VF, int CT, int WC, int WK, bool KV> void launch_attention(hipStream_t s, const StackAttn & a) {
    constexpr int lds = WK * 2 * (KF + (KV ? VF : 0)) * 2048;
    auto kernel = k_stack_attention<KF, VF, CT, WC, WK, KV>;
    static const bool allowed = hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, lds) == hipSuccess;
    if (!allowed) throw std::runtime_error("attention: the page buffers do not fit the LDS");
    hipLaunchKernelGGL(kernel, dim3((unsigned)a.n_blocks, (unsigned)a.splits, (unsigned)a.G), dim3(64 * WC * WK), lds, s, a);
}
template <int KF, int VF, bool KV> void launch_columns(hipStream_t s, const StackAttn & a) {
    switch (a.block_cols) {
        case 16: launch_attention<KF, VF, 1, 1, 2, KV>(s, a); break;
        case 32: launch_attention<KF, VF, 1, 2, 2, KV>(s, a); break;
        case 64: launch_attention<KF, VF, 1, 4, 1, KV>(s, a); break;
        case 128:
            if constexpr (KF <= 8) { launch_attention<KF, VF, 2, 4, 1, KV>(s, a); break; }      // wider: the registers do not suffice
            [[fallthrough]];
        default: throw std::runtime_error("attention: no kernel for this many columns per block");
    }
}
template <int I = 0> void launch_pair(hipStream_t s, const StackAttn & a) {
    if constexpr (I < (int)(sizeof(kPairs) / sizeof(kPairs[0]))) {
        if (a.kf == kPairs[I].k && a.vf == kPairs[I].v) return launch_columns<kPairs[I].k, kPairs[I].v, true>(s, a);
        launch_pair<I + 1>(s, a);
    } else {
        throw std::runtime_error("attention: no kernel for this pair of cache widths");
    }
}
template <bool KV> void launch_width(hipStream_t s, const StackAttn & a) {
    switch (a.kf) {                   // the widths cache_frags() rounds to
        case 1: return launch_columns<1, 1, KV>(s, a);
        case 2: return launch_columns<2, 2, KV>(s, a);
        case 3: return launch_columns<3, 3, KV>(s, a);
        case 4: return launch_columns<4, 4, KV>(s, a);
        case 6: return launch_columns<6, 6, KV>(s, a);
        case 8: return launch_columns<8, 8, KV>(s, a);
        case 12: if constexpr (!KV) return launch_columns<12, 12, KV>(s, a); break;
        case 16: if constexpr (!KV) return launch_columns<16, 16, KV>(s, a); break;
        default: break;
    }
    throw std::runtime_error("attention: no kernel for this cache width");
}
}  // namespace

int cache_frags(int kv_rank) {
    const int kf = frags_of(kv_rank);
    for (int w : {1, 2, 3, 4, 6, 8, 12, 16}) if (kf <= w) return w;
    return kf;
}

PairFrags pair_frags(int key_columns, int value_columns) {
    const int k = frags_of(key_columns), v = frags_of(value_columns), both = std::max(k, v);
    if (both > kMatrixKfPair) return {k, v};
    PairFrags best = {cache_frags(both * 32), cache_frags(both * 32)};
    for (const PairFrags & p : kPairs)
        if (k <= p.k && v <= p.v && p.k + p.v < best.k + best.v) best = p;
    return best;
}

int stack_block_cols(int arith, int cols_per_token, int kf, int vf, bool pair, int n_tokens, int n_rows) {
    if (!on_matrix_cores(arith, kf, vf, pair)) return 1;
    if (n_tokens == n_rows) return cols_per_token <= 16 ? 16 : cols_per_token <= 32 ? 32 : 64;      // one token per row
    return std::max(kf, vf) <= 8 && (int64_t)n_tokens * cols_per_token >= 256 * 128 ? 128 : 64;
}

int stack_splits(int arith, const StackAttn & a, int max_resident) {
    if (!on_matrix_cores(arith, a.kf, a.vf, a.v_pool)) return 1;
    const int reach = a.chunk > 0 ? a.chunk : a.window, keys = reach > 0 ? std::min(reach, max_resident) : max_resident;
    const int pages = (keys + PAGE - 1) / PAGE + 1, per = a.block_cols <= 32 ? 2 : 1;
    return std::max(1, std::min({256 / std::max(a.n_blocks * a.G, 1), pages / per, 32}));
}

size_t stack_partial_floats(int T, int H, int vf, int splits) { return splits > 1 ? (size_t)T * H * splits * (vf * 16 + 2) : 0; }

void stack_attention(hipStream_t s, int arith, const StackAttn & a) {
    if (a.n_blocks <= 0) return;
    if (std::max(a.kf, a.vf) * 32 > 1024) throw std::runtime_error("attention: cache rows of at most 1024 columns per head");
    if (on_matrix_cores(arith, a.kf, a.vf, a.v_pool)) {
        if (a.v_pool && a.kf != a.vf) launch_pair(s, a);
        else if (a.v_pool) launch_width<true>(s, a);
        else launch_width<false>(s, a);
        check_launch("stack_attention");
        return;
    }
    const size_t lds = ((size_t)a.kf * 32 + 256) * 4;
    const dim3 grid((unsigned)a.n_blocks, (unsigned)a.G);
    if (arith == ARITH_16) hipLaunchKernelGGL(k_stack_attention_any<ARITH_16>, grid, dim3(256), lds, s, a);
    else hipLaunchKernelGGL(k_stack_attention_any<ARITH_32>, grid, dim3(256), lds, s, a);
    check_launch("stack_attention");
}

void stack_combine(hipStream_t s, const StackAttn & a, int T) {
    if (a.splits <= 1 || T <= 0) return;
    hipLaunchKernelGGL(k_stack_combine, dim3((unsigned)(T * a.H)), dim3(64), 0, s, a);
    check_launch("stack_combine");
}

void stack_copy_page(hipStream_t s, void * pool, size_t page_bytes, int src, int dst) {
    const size_t n = page_bytes / 16;
    hipLaunchKernelGGL(k_copy16, dim3((unsigned)std::min<size_t>((n + 255) / 256, 256)), dim3(256), 0, s,
                       (const u4 *)((const uint8_t *)pool + (size_t)src * page_bytes), (u4 *)((uint8_t *)pool + (size_t)dst * page_bytes), n);
    check_launch("stack_copy_page");
}

void copy_floats(hipStream_t s, const float * src, float * dst, size_t n) {
    if (n == 0) return;
    hipLaunchKernelGGL(k_copy4, dim3((unsigned)std::min<size_t>((n + 255) / 256, 1024)), dim3(256), 0, s, src, dst, n);
    check_launch("copy_floats");
}

void stack_cells(hipStream_t s, void * pool, int kf, int elem, const int32_t * cells, int n, void * rows, bool gather) {
    if (n <= 0) return;
    const int64_t total = (int64_t)n * kf * 4;
    const dim3 grid((unsigned)std::min<int64_t>((total + 255) / 256, 4096));
    if (elem == 2) hipLaunchKernelGGL(k_stack_cells<uint16_t>, grid, dim3(256), 0, s, (uint16_t *)pool, kf, cells, n, (uint16_t *)rows, gather);
    else hipLaunchKernelGGL(k_stack_cells<uint32_t>, grid, dim3(256), 0, s, (uint32_t *)pool, kf, cells, n, (uint32_t *)rows, gather);
    check_launch("stack_cells");
}

}  // namespace rk
