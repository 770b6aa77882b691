// Routing of mixture-of-experts feed-forwards of layer-stack models: the choice of experts per token and the order in
// which the expert products (dense.hip) take the chosen pairs. Logits arrive in f32; the weights of a token are the
// softmax over its chosen logits, over all its logits, or each logit's own sigmoid.
#include "stack_dev.hpp"

namespace rk {

namespace {

// Logits of experts outside the kept groups become -infinity: a group's rank is the number of groups whose largest logit
// comes before its own (ties to the lower group).
template <int N> __device__ __forceinline__ void keep_groups(const ExpertRoute & r, int lane, float (&v)[N]) {
    const int size = r.experts / r.groups;
    float best[N];                              // of the lane's experts' groups
    int own[N], rank[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
        own[i] = (lane + 64 * i) / size;
        best[i] = -INFINITY;
        rank[i] = 0;
    }
    auto best_of = [&](int g) {
        float m = -INFINITY;
#pragma unroll
        for (int i = 0; i < N; ++i) m = own[i] == g ? fmaxf(m, v[i]) : m;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o, 64));
        return m;
    };
#pragma unroll 1
    for (int g = 0; g < r.groups; ++g) {
        const float m = best_of(g);
#pragma unroll
        for (int i = 0; i < N; ++i) best[i] = own[i] == g ? m : best[i];
    }
#pragma unroll 1
    for (int g = 0; g < r.groups; ++g) {
        const float m = best_of(g);
#pragma unroll
        for (int i = 0; i < N; ++i) rank[i] += m > best[i] || (m == best[i] && g < own[i]) ? 1 : 0;
    }
#pragma unroll
    for (int i = 0; i < N; ++i) if (rank[i] >= r.keep) v[i] = -INFINITY;
}

// One wave: the experts of token t, lane l holding the logits of experts l + 64 i. Every expert's rank is the number of
// logits before its own; rank j < top is choice j.
template <int N> __device__ __forceinline__ void choose(const ExpertRoute & r, int t, int lane, int32_t * sel) {
    const float * z = r.logits + (size_t)t * r.ld;
    float v[N], largest = -INFINITY;
    int rank[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const int e = lane + 64 * i;
        v[i] = e < r.experts ? fmaxf(z[e], -3.4e38f) : -INFINITY;      // any order is a total one: no NaN, and open places come last
        rank[i] = 0;
        largest = fmaxf(largest, v[i]);
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) largest = fmaxf(largest, __shfl_xor(largest, o, 64));
    float sum = 0.0f;
    if (r.score == SCORE_OVER_ALL) {
#pragma unroll
        for (int i = 0; i < N; ++i) sum += expf(v[i] - largest);
    }
    if (r.groups > 1) keep_groups<N>(r, lane, v);
#pragma unroll 8
    for (int o = 0; o < 64; ++o) {
#pragma unroll
        for (int j = 0; j < N; ++j) {
            const float other = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v[j]), o));
#pragma unroll
            for (int i = 0; i < N; ++i) rank[i] += other > v[i] || (other == v[i] && (j < i || (j == i && o < lane))) ? 1 : 0;
        }
    }
    float p[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
        p[i] = rank[i] < r.top ? expf(v[i] - largest) : 0.0f;
        if (r.score == SCORE_OVER_CHOSEN) sum += p[i];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int i = 0; i < N; ++i)
        if (rank[i] < r.top) {
            sel[rank[i]] = lane + 64 * i;
            r.weight[(size_t)t * r.top + rank[i]] = (r.score == SCORE_SIGMOID ? sigmoid_f(v[i]) : p[i] / sum) * r.scale;
        }
}
__device__ __forceinline__ void choose_any(const ExpertRoute & r, int t, int lane, int32_t * sel) {
    if (r.experts <= 64) choose<1>(r, t, lane, sel);
    else if (r.experts <= 128) choose<2>(r, t, lane, sel);
    else if (r.experts <= 256) choose<4>(r, t, lane, sel);
    else choose<MAX_EXPERTS / 64>(r, t, lane, sel);
}

// One workgroup of 1024 threads: the pairs' slots and the tiles. The order of an expert's pairs is whatever the atomics
// give; it changes no result, since a pair's column is computed alone.
__device__ __forceinline__ void group(const ExpertRoute & r, const int32_t * sel, int n_pairs) {
    __shared__ int count[MAX_EXPERTS], base[MAX_EXPERTS], part[2][16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    count[tid] = 0;
    __syncthreads();
    for (int p = tid; p < n_pairs; p += 1024) atomicAdd(&count[sel[p]], 1);
    __syncthreads();
    const int n = count[tid], padded = (n + 15) / 16 * 16, tiles = (n + r.block - 1) / r.block;
    int a = padded, b = tiles;                  // inclusive sums over the wave, then over the waves
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const int x = __shfl_up(a, o, 64), y = __shfl_up(b, o, 64);
        if (lane >= o) { a += x; b += y; }
    }
    if (lane == 63) { part[0][wave] = a; part[1][wave] = b; }
    __syncthreads();
    for (int w = 0; w < wave; ++w) { a += part[0][w]; b += part[1][w]; }
    base[tid] = a - padded;
    if (tid == MAX_EXPERTS - 1) *r.n_tiles = b;
    for (int i = 0; i < tiles; ++i)
        ((int4 *)r.tiles)[b - tiles + i] = make_int4(tid, a - padded + i * r.block, min(r.block, n - i * r.block), 0);
    __syncthreads();
    for (int p = tid; p < n_pairs; p += 1024) r.slot_pair[atomicAdd(&base[sel[p]], 1)] = p;
}

__global__ __launch_bounds__(256) void k_expert_choose(ExpertRoute r, int T) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < T) choose_any(r, t, threadIdx.x & 63, r.sel + (size_t)t * r.top);
}
__global__ __launch_bounds__(1024) void k_expert_group(ExpertRoute r, int n_pairs) { group(r, r.sel, n_pairs); }
// Short steps: both in one launch, the choices in LDS.
constexpr int ONE_LAUNCH_TOKENS = 16;
__global__ __launch_bounds__(1024) void k_expert_route(ExpertRoute r, int T) {
    __shared__ int32_t sel[ONE_LAUNCH_TOKENS * MAX_TOP];
    const int t = threadIdx.x >> 6;               // a wave per token
    if (t < T) choose_any(r, t, threadIdx.x & 63, sel + t * r.top);
    __syncthreads();
    group(r, sel, T * r.top);
}

}  // namespace

size_t expert_slots(int T, int top, int experts) {
    const size_t pairs = (size_t)T * top;
    return pairs + 15 * std::min<size_t>(pairs, (size_t)experts) + 128;
}

int expert_max_tiles(int T, int top, int experts, int block) {
    const int64_t pairs = (int64_t)T * top, partial = std::min<int64_t>(pairs, experts);
    return (int)std::min<int64_t>(pairs, partial + (pairs - partial) / block);
}

void expert_route(hipStream_t s, const ExpertRoute & r, int T) {
    if (T <= 0) return;
    if (r.experts > MAX_EXPERTS || r.top > MAX_TOP || r.top > r.experts || r.groups < 1 || r.experts % r.groups != 0 || r.keep < 1
            || (r.groups > 1 && (int64_t)r.keep * (r.experts / r.groups) < r.top)) throw std::runtime_error("expert routing: unsupported sizes");
    if (T <= ONE_LAUNCH_TOKENS) {
        hipLaunchKernelGGL(k_expert_route, dim3(1), dim3(1024), 0, s, r, T);
    } else {
        hipLaunchKernelGGL(k_expert_choose, dim3((unsigned)((T + 3) / 4)), dim3(256), 0, s, r, T);
        hipLaunchKernelGGL(k_expert_group, dim3(1), dim3(1024), 0, s, r, T * r.top);
    }
    check_launch("expert_route");
}

}  // namespace rk
