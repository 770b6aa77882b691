// Routing of mixture-of-experts feed-forwards of layer-stack models: the choice of experts per token and the order in
// which the expert products (dense.hip) take the chosen pairs. Logits arrive in f32; the weights of a token are the
// softmax over its chosen logits.
#include "stack_dev.hpp"

namespace rk {

namespace {

constexpr int PER_LANE = MAX_EXPERTS / 64;

// One wave: the experts of token t.
__device__ __forceinline__ void choose(const ExpertRoute & r, int t, int lane) {
    const float * z = r.logits + (size_t)t * r.ld;
    float v[PER_LANE];
    bool open[PER_LANE];
#pragma unroll
    for (int i = 0; i < PER_LANE; ++i) {
        const int e = lane + 64 * i;
        open[i] = e < r.experts;
        v[i] = open[i] ? z[e] : 0.0f;
    }
    const int n = (r.experts + 63) / 64;
    float mine = -INFINITY;                     // lane j: the j-th largest logit
    float largest = 0.0f;
    for (int j = 0; j < r.top; ++j) {
        float best = 0.0f;
        int at = -1;
#pragma unroll
        for (int i = 0; i < PER_LANE; ++i)
            if (i < n && open[i] && (at < 0 || v[i] > best)) { best = v[i]; at = lane + 64 * i; }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float b = __shfl_xor(best, o, 64);
            const int a = __shfl_xor(at, o, 64);
            if (a >= 0 && (at < 0 || b > best || (b == best && a < at))) { best = b; at = a; }
        }
#pragma unroll
        for (int i = 0; i < PER_LANE; ++i) if (at == lane + 64 * i) open[i] = false;
        if (j == 0) largest = best;
        if (lane == j) { mine = best; r.sel[(size_t)t * r.top + j] = at; }
    }
    const float p = lane < r.top ? expf(mine - largest) : 0.0f;
    const float sum = wave_sum(p);
    if (lane < r.top) r.weight[(size_t)t * r.top + lane] = p / sum;
}

// One workgroup of 1024 threads: the pairs' slots and the tiles. The order of an expert's pairs is whatever the atomics
// give; it changes no result, since a pair's column is computed alone.
__device__ void group(const ExpertRoute & r, int n_pairs) {
    __shared__ int count[MAX_EXPERTS], base[MAX_EXPERTS], part[2][16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    count[tid] = 0;
    __syncthreads();
    for (int p = tid; p < n_pairs; p += 1024) atomicAdd(&count[r.sel[p]], 1);
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
    for (int p = tid; p < n_pairs; p += 1024) r.slot_pair[atomicAdd(&base[r.sel[p]], 1)] = p;
}

__global__ __launch_bounds__(256) void k_expert_choose(ExpertRoute r, int T) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < T) choose(r, t, threadIdx.x & 63);
}
__global__ __launch_bounds__(1024) void k_expert_group(ExpertRoute r, int n_pairs) { group(r, n_pairs); }
// Short steps: both in one launch.
__global__ __launch_bounds__(1024) void k_expert_route(ExpertRoute r, int T) {
    for (int t = threadIdx.x >> 6; t < T; t += 16) choose(r, t, threadIdx.x & 63);
    __threadfence_block();
    __syncthreads();
    group(r, T * r.top);
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
    if (r.experts > MAX_EXPERTS || r.top > MAX_TOP || r.top > r.experts) throw std::runtime_error("expert routing: too many experts");
    if (T <= 64) {
        hipLaunchKernelGGL(k_expert_route, dim3(1), dim3(1024), 0, s, r, T);
    } else {
        hipLaunchKernelGGL(k_expert_choose, dim3((unsigned)((T + 3) / 4)), dim3(256), 0, s, r, T);
        hipLaunchKernelGGL(k_expert_group, dim3(1), dim3(1024), 0, s, r, T * r.top);
    }
    check_launch("expert_route");
}

}  // namespace rk
