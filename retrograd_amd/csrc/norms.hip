// Row norms of layer-stack models: the residual stream (completed with the slices the products before left), or what a
// sublayer reads of several residual streams, through an RMS or layer norm into activations; norms in groups before and after
// a sublayer with the convolution of what it reads. Statistics in f32, two passes over the row held in LDS. Also the rows that
// start a stream.
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

// Norms in `groups` equal parts of a row of E columns held in LDS: its floats, then a factor per group and the partial sums.
struct GroupNorm {
    float * row, * inv, * part;
    int E, groups, len;
    float eps;
    __device__ __forceinline__ GroupNorm(float * lds, int E, int groups, float eps)
        : row(lds), inv(lds + (E + 3) / 4 * 4), part(inv + groups), E(E), groups(groups), len(E / groups), eps(eps) {}
    // The factors of what the row holds. Waves share a group where there are fewer groups than waves.
    __device__ __forceinline__ void factors() {
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6, per = max(1, waves / groups);
        const bool even = len % (4 * per) == 0;
        __syncthreads();
        for (int i = wave; i < groups * per; i += waves) {
            const int g = i / per, p = i - g * per, lo = g * len + (int)((int64_t)len * p / per), hi = g * len + (int)((int64_t)len * (p + 1) / per);
            float q = 0.0f;
            if (even) {
                for (int k = lo + 4 * lane; k < hi; k += 256) {
                    const f4 v = *(const f4 *)(row + k);
                    q += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
                }
            } else {
                for (int k = lo + lane; k < hi; k += 64) q += row[k] * row[k];
            }
            q = wave_sum(q);
            if (lane == 0) part[i] = q;
        }
        __syncthreads();
        for (int g = threadIdx.x; g < groups; g += blockDim.x) {
            float q = 0.0f;
            for (int p = 0; p < per; ++p) q += part[g * per + p];
            inv[g] = 1.0f / sqrtf(q / (float)len + eps);
        }
        __syncthreads();
    }
    static size_t bytes(int E, int groups) { return ((size_t)(E + 3) / 4 * 4 + groups + std::max(groups, 16)) * 4; }
};

// Where a sublayer's input goes: activations at once, f32 rows for the convolution that follows, or through the convolution
// where every run is a single token (a workgroup per run).
enum : int { NORM_TO_ACT = 0, NORM_TO_ROWS, NORM_CONVOLVED };

// W columns (1, or 4 from a multiple of 4) of a row as activations from element `at` on.
template <int ARITH, typename VEC> __device__ __forceinline__ void store_columns(void * act, size_t at, const VEC & v) {
    if constexpr (sizeof(VEC) == 4) {
        if constexpr (ARITH == ARITH_16) ((uint16_t *)act)[at] = bf16_bits(v[0]);
        else ((float *)act)[at] = v[0];
    } else if constexpr (ARITH == ARITH_16) {
        uint2 u;
        u.x = (uint32_t)bf16_bits(v[0]) | ((uint32_t)bf16_bits(v[1]) << 16);
        u.y = (uint32_t)bf16_bits(v[2]) | ((uint32_t)bf16_bits(v[3]) << 16);
        *(uint2 *)((uint16_t *)act + at) = u;
    } else {
        *(VEC *)((float *)act + at) = v;
    }
}

// A thread holds W columns, NV times, from the reads to the writes; everything that does not hang on a norm is requested at
// the start. WAVES: a group is whole steps of a wave, whose sums are all that goes through LDS.
template <int ARITH, int OUT, int W, int NV, bool WAVES>
__global__ __launch_bounds__(1024) void k_sublayer_norm(SublayerNorm j) {
    typedef float vec __attribute__((ext_vector_type(W)));
    constexpr int PAST = NV <= 2 ? 3 : 0;         // inputs from earlier steps that are requested at the start
    extern __shared__ __attribute__((aligned(16))) float sm[];
    GroupNorm norm(sm, j.E, j.groups, j.eps);
    const int E = j.E, n_thr = blockDim.x, wave = threadIdx.x >> 6, waves = n_thr >> 6;
    SeqRun run = {};
    if constexpr (OUT == NORM_CONVOLVED) run = j.runs.runs[blockIdx.x];
    const int t = OUT == NORM_CONVOLVED ? j.runs.tok[run.start] : j.rows ? j.rows[blockIdx.x] : (int)blockIdx.x;
    const int at = OUT == NORM_CONVOLVED ? t : (int)blockIdx.x;              // row of the activations
    const int past = OUT == NORM_CONVOLVED ? j.n_taps - 1 : 0, plane = (run.flags >> 1) & 1;
    const bool fresh = run.flags & 1;
    const float * old_in = nullptr;
    float * new_in = nullptr;
    if constexpr (OUT == NORM_CONVOLVED) {
        old_in = j.history + (size_t)plane * j.plane + (size_t)run.slot * past * E;
        new_in = j.history + (size_t)(1 - plane) * j.plane + (size_t)run.slot * past * E;
    }
    float * xr = j.x + (size_t)t * E;
    auto column = [&](int i) { return W * ((int)threadIdx.x + n_thr * i); };
    auto remembered = [&](int p, int k) { return fresh ? vec(0.0f) : *(const vec *)(old_in + (size_t)p * E + k); };
    vec x[NV], y[NV], w[NV], tap[NV], held[NV][PAST + 1], taps[NV][PAST + 1];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int k = column(i);
        x[i] = y[i] = w[i] = vec(0.0f);
        if (k >= E) continue;
        x[i] = *(const vec *)(xr + k);
        for (int base = 0; base < j.add.n; base += 8) {
            const float * from = j.add.data + (size_t)base * j.add.stride + (size_t)t * E + k;
            const int n = j.add.n - base;
            vec d[8];
#pragma unroll
            for (int s = 0; s < 8; ++s) if (s < n) d[s] = *(const vec *)(from + (size_t)s * j.add.stride);
#pragma unroll
            for (int s = 0; s < 8; ++s) if (s < n) y[i] += d[s];
        }
        if (j.w) w[i] = *(const vec *)(j.w + k);
        if constexpr (OUT == NORM_CONVOLVED) {
            tap[i] = *(const vec *)(j.taps + (size_t)past * E + k);
#pragma unroll
            for (int p = 0; p < PAST; ++p)
                if (p < past) {
                    held[i][p] = remembered(p, k);
                    taps[i][p] = *(const vec *)(j.taps + (size_t)p * E + k);
                }
        }
    }
    auto factors = [&](const vec (&v)[NV], int turn, float (&inv)[NV]) {
        if constexpr (WAVES) {
            float * part = sm + turn * NV * waves;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                float q = 0.0f;
#pragma unroll
                for (int e = 0; e < W; ++e) q += v[i][e] * v[i][e];
                q = wave_sum(q);
                if ((threadIdx.x & 63) == 0) part[i * waves + wave] = q;
            }
            __syncthreads();
            const int per = norm.len / (64 * W);
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                if (column(i) >= E) continue;
                const int first = (i * waves + wave) / per * per;
                float q = 0.0f;
                for (int p = 0; p < per; ++p) q += part[first + p];
                inv[i] = 1.0f / sqrtf(q / (float)norm.len + j.eps);
            }
        } else {
#pragma unroll
            for (int i = 0; i < NV; ++i) if (column(i) < E) *(vec *)(norm.row + column(i)) = v[i];
            norm.factors();
#pragma unroll
            for (int i = 0; i < NV; ++i) if (column(i) < E) inv[i] = norm.inv[column(i) / norm.len];
        }
    };
    float inv[NV];
    if (j.add.n > 0) {
        if (j.after) factors(y, 0, inv);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int k = column(i);
            if (k >= E) continue;
            if (j.after) y[i] = y[i] * inv[i] * *(const vec *)(j.after + k);
            x[i] += j.mult * y[i];
            if (!j.rows) *(vec *)(xr + k) = x[i];
        }
    }
    if (!j.w) return;
    factors(x, 1, inv);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int k = column(i);
        if (k >= E) continue;
        const vec h = x[i] * inv[i] * w[i];
        if constexpr (OUT == NORM_TO_ROWS) {
            *(vec *)(j.h + (size_t)t * E + k) = h;
            continue;
        }
        vec v = h;
        if constexpr (OUT == NORM_CONVOLVED) {
            v += tap[i] * h;
            auto take = [&](int p, const vec & o, const vec & f) {
                v += f * o;
                if (p > 0) *(vec *)(new_in + (size_t)(p - 1) * E + k) = o;
            };
#pragma unroll
            for (int p = 0; p < PAST; ++p) if (p < past) take(p, held[i][p], taps[i][p]);
            for (int p = PAST; p < past; ++p) take(p, remembered(p, k), *(const vec *)(j.taps + (size_t)p * E + k));
            if (past > 0) *(vec *)(new_in + (size_t)(past - 1) * E + k) = h;
        }
        store_columns<ARITH>(j.act, frag_at(at, k, j.act_kf), v);
        if (j.act_rows) store_columns<ARITH>(j.act_rows, (size_t)at * j.act_kf * 32 + k, v);
    }
}

// The convolution over the rows k_sublayer_norm left: a wave takes 16 tokens of a run and 32 columns, a lane eight columns of one
// token, so that reads are whole cache lines and a wave's activations one fragment (TAPS 0: any number).
template <int ARITH, int TAPS>
__global__ __launch_bounds__(256) void k_sublayer_conv(SublayerNorm j) {
    const int E = j.E, K = TAPS > 0 ? TAPS : j.n_taps, lane = threadIdx.x & 63;
    const int k = ((int)blockIdx.x * 4 + (threadIdx.x >> 6)) * 32 + 8 * (lane >> 4), i = blockIdx.y * 16 + (lane & 15), left = E - k;
    const SeqRun run = j.runs.runs[blockIdx.z];
    if (left <= 0 || i >= run.n) return;
    const int plane = (run.flags >> 1) & 1;
    const bool even = E % 4 == 0;
    const float * old_in = j.history + (size_t)plane * j.plane + (size_t)run.slot * (K - 1) * E + k;
    float * new_in = j.history + (size_t)(1 - plane) * j.plane + (size_t)run.slot * (K - 1) * E + k;
    const int32_t * tok = j.runs.tok + run.start;
    auto load = [&](const float * p, float (&o)[8]) {
        if (even && left >= 8) {
            const f4 a = *(const f4 *)p, b = *(const f4 *)(p + 4);
#pragma unroll
            for (int e = 0; e < 4; ++e) { o[e] = a[e]; o[4 + e] = b[e]; }
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = e < left ? p[e] : 0.0f;
        }
    };
    auto input = [&](int at, float (&o)[8]) {        // of the run's token `at`; below 0: what the slot remembers
        if (at >= 0) return load(j.h + (size_t)tok[at] * E + k, o);
        if (!(run.flags & 1)) return load(old_in + (size_t)(at + K - 1) * E, o);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = 0.0f;
    };
    auto remember = [&](int p, const float (&o)[8]) {
#pragma unroll
        for (int e = 0; e < 8; ++e) if (e < left) new_in[(size_t)p * E + e] = o[e];
    };
    const int t = tok[i];
    float h[8], v[8];
    load(j.h + (size_t)t * E + k, h);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = h[e];
#pragma unroll TAPS > 0 ? TAPS : 1
    for (int p = 0; p < K; ++p) {
        float o[8], w[8];
        input(i - (K - 1) + p, o);
        load(j.taps + (size_t)p * E + k, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] += w[e] * o[e];
    }
    store_frag8<ARITH>(j.act, j.act_kf, t, k, v);
    if (j.act_rows) store_act8_at<ARITH>(j.act_rows, (size_t)t * j.act_kf * 32 + k, v);
    // the run's last inputs stay; a short run's first lane moves what is older
    const int from = run.n - (K - 1);
    if (i >= from) remember(i - from, h);
    if (i == 0)
        for (int p = 0; p < -from; ++p) {
            input(from + p, h);
            remember(p, h);
        }
}

// One workgroup per token of a run.
__global__ __launch_bounds__(256) void k_embed_pairs(PairEmbedding j) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const SeqRun run = j.runs.runs[blockIdx.y];
    const int i = blockIdx.x;
    if (i >= run.n) return;
    GroupNorm norm(sm, j.E, j.groups, j.eps);
    const int plane = (run.flags >> 1) & 1, t = j.runs.tok[run.start + i], tok = j.tok[t];
    int64_t pair = j.buckets;
    if (i > 0 || !(run.flags & 1)) {
        const int before = i > 0 ? j.tok[j.runs.tok[run.start + i - 1]] : (int)j.last[(size_t)plane * j.plane + run.slot];
        pair = (before * j.mul_prev + tok * j.mul_cur) % j.buckets;
    }
    const uint16_t * e = j.embed + (size_t)tok * j.E, * p = j.pairs + (size_t)pair * j.E;
    float * x = j.x + (size_t)t * j.E;
    if (j.E % 8 == 0) {
        for (int k = 8 * (int)threadIdx.x; k < j.E; k += 8 * 256) {
            const u4 a = *(const u4 *)(e + k), b = *(const u4 *)(p + k);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                norm.row[k + 2 * i] = bf16_float((uint16_t)a[i]) * j.scale + bf16_float((uint16_t)b[i]);
                norm.row[k + 2 * i + 1] = bf16_float((uint16_t)(a[i] >> 16)) * j.scale + bf16_float((uint16_t)(b[i] >> 16));
            }
        }
    } else {
        for (int k = threadIdx.x; k < j.E; k += 256) norm.row[k] = bf16_float(e[k]) * j.scale + bf16_float(p[k]);
    }
    norm.factors();
    if (norm.len % 4 == 0) {
        for (int k = 4 * (int)threadIdx.x; k < j.E; k += 4 * 256) *(f4 *)(x + k) = *(const f4 *)(norm.row + k) * norm.inv[k / norm.len] * *(const f4 *)(j.w + k);
    } else {
        for (int k = threadIdx.x; k < j.E; k += 256) x[k] = norm.row[k] * norm.inv[k / norm.len] * j.w[k];
    }
    if (i == run.n - 1 && threadIdx.x == 0) j.last[(size_t)(1 - plane) * j.plane + run.slot] = (float)tok;      // exact: a vocabulary has at most 2^24 tokens
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

void sublayer_norm(hipStream_t s, int arith, const SublayerNorm & n, int n_rows) {
    if (n_rows <= 0) return;
    if (n.groups < 1 || n.E % n.groups != 0) throw std::runtime_error("norm: the row does not split into its groups");
    const bool conv = n.taps && n.w;
    const int out = !conv ? NORM_TO_ACT : n.runs.longest <= 1 ? NORM_CONVOLVED : NORM_TO_ROWS;
    const int len = n.E / n.groups, width = len % 4 == 0 ? 4 : 1;
    const bool waves = len % 256 == 0;
    // few rows: a column group per thread; many: fewer waves to wait for one another
    int threads = n_rows <= 512 ? std::min(1024, (n.E / width + 63) / 64 * 64) : 256;
    if (n.E > 16 * width * threads) threads = 1024;
    const int steps = (n.E + width * threads - 1) / (width * threads);
    auto go = [&](auto kernel) {
        hipLaunchKernelGGL(kernel, dim3((unsigned)(out == NORM_CONVOLVED ? n.runs.n : n_rows)), dim3((unsigned)threads), GroupNorm::bytes(n.E, n.groups), s, n);
        check_launch("sublayer_norm");
    };
    auto step = [&](auto arithmetic, auto kind, auto w, auto whole) {
        constexpr int A = decltype(arithmetic)::value, O = decltype(kind)::value, W = decltype(w)::value;
        constexpr bool V = decltype(whole)::value;
        if (steps <= 1) go(k_sublayer_norm<A, O, W, 1, V>);
        else if (steps <= 2) go(k_sublayer_norm<A, O, W, 2, V>);
        else if (steps <= 4) go(k_sublayer_norm<A, O, W, 4, V>);
        else if (steps <= 16) go(k_sublayer_norm<A, O, W, 16, V>);
        else throw std::runtime_error("norm: rows this wide are not supported");
    };
    auto columns = [&](auto arithmetic, auto kind) {
        if (waves) step(arithmetic, kind, std::integral_constant<int, 4>(), std::true_type());
        else if (width == 4) step(arithmetic, kind, std::integral_constant<int, 4>(), std::false_type());
        else step(arithmetic, kind, std::integral_constant<int, 1>(), std::false_type());
    };
    auto kinds = [&](auto arithmetic) {
        if (out == NORM_TO_ACT) columns(arithmetic, std::integral_constant<int, NORM_TO_ACT>());
        else if (out == NORM_TO_ROWS) columns(arithmetic, std::integral_constant<int, NORM_TO_ROWS>());
        else columns(arithmetic, std::integral_constant<int, NORM_CONVOLVED>());
    };
    if (arith == ARITH_16) kinds(std::integral_constant<int, ARITH_16>());
    else kinds(std::integral_constant<int, ARITH_32>());
    if (out != NORM_TO_ROWS) return;
    const dim3 grid((unsigned)((n.E + 127) / 128), (unsigned)((n.runs.longest + 15) / 16), (unsigned)n.runs.n);
    auto taps = [&](auto arithmetic) {
        constexpr int A = decltype(arithmetic)::value;
        switch (n.n_taps) {
            case 2: hipLaunchKernelGGL((k_sublayer_conv<A, 2>), grid, dim3(256), 0, s, n); break;
            case 3: hipLaunchKernelGGL((k_sublayer_conv<A, 3>), grid, dim3(256), 0, s, n); break;
            case 4: hipLaunchKernelGGL((k_sublayer_conv<A, 4>), grid, dim3(256), 0, s, n); break;
            default: hipLaunchKernelGGL((k_sublayer_conv<A, 0>), grid, dim3(256), 0, s, n);
        }
    };
    if (arith == ARITH_16) taps(std::integral_constant<int, ARITH_16>());
    else taps(std::integral_constant<int, ARITH_32>());
    check_launch("sublayer_conv");
}

void embed_pairs(hipStream_t s, const PairEmbedding & e, int T) {
    if (T <= 0 || e.runs.n <= 0) return;
    if (e.groups < 1 || e.E % e.groups != 0 || e.buckets < 1) throw std::runtime_error("embedding: unsupported sizes");
    hipLaunchKernelGGL(k_embed_pairs, dim3((unsigned)e.runs.longest, (unsigned)e.runs.n), dim3(256), GroupNorm::bytes(e.E, e.groups), s, e);
    check_launch("embed_pairs");
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
