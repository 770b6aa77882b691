// The Mamba-2 mixer between its two projections: short causal convolution with SiLU over x, B and C, the state-space
// recurrence per head, and the gated grouped RMS norm. Everything here is f32 in both arithmetics; only the rows that
// leave for the output projection take the arithmetic's activation type.
#include "stack_dev.hpp"

namespace rk {

namespace {

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

constexpr int kConvTokens = 16;       // tokens of a run one workgroup convolves

// xbc[t][c] = silu(bias + sum over the taps); inputs before the run come from the slot's current plane, and the run's
// last taps - 1 inputs go to the other plane (the workgroups of a run read the one while the other is written).
__global__ __launch_bounds__(256) void k_mamba_conv(MambaJob j) {
    const MambaShape sh = j.sh;
    const int C = sh.channels(), c = blockIdx.y * 256 + threadIdx.x, K = sh.taps;
    const SeqRun run = j.runs[blockIdx.z];
    const int first = blockIdx.x * kConvTokens;
    if (c >= C || first >= run.n) return;
    const int plane = (run.flags >> 1) & 1;
    const bool fresh = run.flags & 1;
    const float * old_in = j.conv_state + (size_t)plane * j.conv_plane + (size_t)run.slot * (K - 1) * C;
    float * new_in = j.conv_state + (size_t)(1 - plane) * j.conv_plane + (size_t)run.slot * (K - 1) * C;
    const int off = sh.inner() + c;
    auto input = [&](int i) -> float {          // input of the run's token i; i < 0: what the slot remembers
        if (i >= 0) return j.proj[(size_t)j.run_tok[run.start + i] * j.ld + off];
        return fresh ? 0.0f : old_in[(size_t)(i + K - 1) * C + c];
    };
    const float * w = j.conv_w + (size_t)c * K;
    const int last = min(first + kConvTokens, run.n);
    for (int i = first; i < last; ++i) {
        float s = 0.0f;
        for (int k = 0; k < K; ++k) s += w[k] * input(i - (K - 1) + k);
        j.xbc[(size_t)j.run_tok[run.start + i] * C + c] = silu_f(s + j.conv_b[c]);
    }
    if (last == run.n)
        for (int k = 0; k < K - 1; ++k) new_in[(size_t)k * C + c] = input(run.n - (K - 1) + k);
}

constexpr int kScanP = 64;            // columns of the state one workgroup holds
constexpr int kScanTokens = 8;        // tokens staged at once

// The recurrence token by token: thread (p, q) holds the state of column p for rows q, q + 4, ...
template <int NPT>
__global__ __launch_bounds__(256) void k_mamba_scan(MambaJob j) {
    extern __shared__ float sm[];
    const MambaShape sh = j.sh;
    const int N = sh.state, P = sh.vdim, C = sh.channels();
    const int h = blockIdx.x, g = h / (sh.heads / sh.groups);
    const int p = blockIdx.y * kScanP + (threadIdx.x & 63), q = threadIdx.x >> 6;
    const SeqRun run = j.runs[blockIdx.z];
    float * sB = sm, * sC = sB + kScanTokens * N, * part = sC + kScanTokens * N;      // part [tokens][4][64]
    __shared__ float s_dt[kScanTokens], s_decay[kScanTokens];
    const bool mine = p < P;
    float * st = j.state + (((size_t)run.slot * sh.heads + h) * N) * P + p;
    float S[NPT];
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = q + 4 * i;
        S[i] = (mine && n < N && !(run.flags & 1)) ? st[(size_t)n * P] : 0.0f;
    }
    const float a = expf(j.A_log[h]), D = j.D[h], bias = j.dt_bias[h];
    for (int base = 0; base < run.n; base += kScanTokens) {
        const int cnt = min(kScanTokens, run.n - base);
        __syncthreads();
        for (int i = threadIdx.x; i < cnt * N; i += 256) {
            const int tk = i / N, n = i % N;
            const float * row = j.xbc + (size_t)j.run_tok[run.start + base + tk] * C + sh.inner() + g * N + n;
            sB[i] = row[0];
            sC[i] = row[(size_t)sh.groups * N];
        }
        if ((int)threadIdx.x < cnt) {
            const float dt = softplus_f(j.proj[(size_t)j.run_tok[run.start + base + threadIdx.x] * j.ld + sh.inner() + C + h] + bias);
            s_dt[threadIdx.x] = dt;
            s_decay[threadIdx.x] = expf(-a * dt);
        }
        __syncthreads();
        for (int tk = 0; tk < cnt; ++tk) {
            const float x = mine ? j.xbc[(size_t)j.run_tok[run.start + base + tk] * C + h * P + p] : 0.0f;
            const float dx = s_dt[tk] * x, dec = s_decay[tk];
            float y = 0.0f;
#pragma unroll
            for (int i = 0; i < NPT; ++i) {
                const int n = q + 4 * i;
                if (n < N) {
                    S[i] = S[i] * dec + sB[tk * N + n] * dx;
                    y += S[i] * sC[tk * N + n];
                }
            }
            part[(tk * 4 + q) * 64 + (threadIdx.x & 63)] = y;
        }
        __syncthreads();
        for (int tk = q; tk < cnt; tk += 4) {
            if (!mine) continue;
            float y = 0.0f;
#pragma unroll
            for (int i = 0; i < 4; ++i) y += part[(tk * 4 + i) * 64 + (threadIdx.x & 63)];
            const int t = j.run_tok[run.start + base + tk];
            j.y[(size_t)t * sh.inner() + h * P + p] = y + D * j.xbc[(size_t)t * C + h * P + p];
        }
    }
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = q + 4 * i;
        if (mine && n < N) st[(size_t)n * P] = S[i];
    }
}

// act[t] = norm over each of the equal parts of (y * silu(z)), times the weight: one workgroup per token and part.
template <int ARITH>
__global__ __launch_bounds__(256) void k_mamba_gate_norm(MambaJob j) {
    extern __shared__ float row[];
    __shared__ float scratch[16];
    const int inner = j.sh.inner(), len = inner / j.sh.norm_groups;
    const int t = blockIdx.x, k0 = blockIdx.y * len;
    const float * y = j.y + (size_t)t * inner + k0, * z = j.proj + (size_t)t * j.ld + k0;
    float q = 0.0f;
    for (int k = threadIdx.x; k < len; k += 256) {
        const float v = y[k] * silu_f(z[k]);
        row[k] = v;
        q += v * v;
    }
    q = block_sum(q, scratch);
    const float inv = 1.0f / sqrtf(q / (float)len + j.eps);
    if (len % 8 == 0 && k0 % 8 == 0) {
        for (int k = 8 * threadIdx.x; k < len; k += 8 * 256) {
            float v[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = row[k + i] * inv * j.norm_w[k0 + k + i];
            store_frag8<ARITH>(j.out, j.out_kf, t, k0 + k, v);
        }
    } else {
        for (int k = threadIdx.x; k < len; k += 256) {
            const float v = row[k] * inv * j.norm_w[k0 + k];
            const size_t at = frag_at(t, k0 + k, j.out_kf);
            if constexpr (ARITH == ARITH_16) ((uint16_t *)j.out)[at] = bf16_bits(v);
            else ((float *)j.out)[at] = v;
        }
    }
}

}  // namespace

size_t mamba_chunk_floats(const MambaShape & sh, int T, int n_seq) { return 0; }

void mamba_mix(hipStream_t s, int arith, const MambaJob & j, int T) {
    if (j.n_runs <= 0 || T <= 0) return;
    const MambaShape & sh = j.sh;
    if (sh.state > 512) throw std::runtime_error("mamba2: at most 512 state rows per head");
    hipLaunchKernelGGL(k_mamba_conv, dim3((unsigned)((j.max_run + kConvTokens - 1) / kConvTokens), (unsigned)((sh.channels() + 255) / 256), (unsigned)j.n_runs),
                       dim3(256), 0, s, j);
    check_launch("mamba_conv");
    const dim3 grid((unsigned)sh.heads, (unsigned)((sh.vdim + kScanP - 1) / kScanP), (unsigned)j.n_runs);
    const size_t lds = (size_t)(2 * kScanTokens * sh.state + kScanTokens * 256) * 4;
    const int npt = (sh.state + 3) / 4;
    if (npt <= 8) hipLaunchKernelGGL(k_mamba_scan<8>, grid, dim3(256), lds, s, j);
    else if (npt <= 16) hipLaunchKernelGGL(k_mamba_scan<16>, grid, dim3(256), lds, s, j);
    else if (npt <= 32) hipLaunchKernelGGL(k_mamba_scan<32>, grid, dim3(256), lds, s, j);
    else if (npt <= 64) hipLaunchKernelGGL(k_mamba_scan<64>, grid, dim3(256), lds, s, j);
    else hipLaunchKernelGGL(k_mamba_scan<128>, grid, dim3(256), lds, s, j);
    check_launch("mamba_scan");
    const dim3 gn((unsigned)T, (unsigned)sh.norm_groups);
    const size_t nl = (size_t)(sh.inner() / sh.norm_groups) * 4;
    if (arith == ARITH_16) hipLaunchKernelGGL(k_mamba_gate_norm<ARITH_16>, gn, dim3(256), nl, s, j);
    else hipLaunchKernelGGL(k_mamba_gate_norm<ARITH_32>, gn, dim3(256), nl, s, j);
    check_launch("mamba_gate_norm");
}

}  // namespace rk
