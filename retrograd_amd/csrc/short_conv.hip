// Short causal convolution with SiLU of recurrent mixers. The inputs a sequence needs from earlier steps lie in two planes
// per slot: a step reads the current one and leaves the run's last inputs in the other, so that the workgroups of a long
// run need no order among themselves.
#include "stack_dev.hpp"

namespace rk {

namespace {

constexpr int kConvTokens = 16;       // tokens of a run one workgroup convolves

template <int TAPS>
__global__ __launch_bounds__(256) void k_short_conv(ShortConv j) {
    const int C = j.channels, c = blockIdx.y * 256 + threadIdx.x, K = TAPS > 0 ? TAPS : j.taps;
    const SeqRun run = j.runs.runs[blockIdx.z];
    const int first = blockIdx.x * kConvTokens;
    if (c >= C || first >= run.n || run.n < j.least) return;
    const int plane = (run.flags >> 1) & 1;
    const bool fresh = run.flags & 1;
    const float * old_in = j.state + (size_t)plane * j.plane + (size_t)run.slot * (K - 1) * C;
    float * new_in = j.state + (size_t)(1 - plane) * j.plane + (size_t)run.slot * (K - 1) * C;
    auto input = [&](int i) -> float {          // input of the run's token i; i < 0: what the slot remembers
        if (i >= 0) return j.in[(size_t)j.runs.tok[run.start + i] * j.ld + c];
        return fresh ? 0.0f : old_in[(size_t)(i + K - 1) * C + c];
    };
    const float * w = j.w + (size_t)c * K;
    const float bias = j.b ? j.b[c] : 0.0f;
    const int last = min(first + kConvTokens, run.n);
    if constexpr (TAPS > 0) {                   // the window and the taps in registers
        float win[TAPS], tap[TAPS];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) {
            tap[k] = w[k];
            win[k] = k > 0 ? input(first - TAPS + k) : 0.0f;
        }
        for (int i = first; i < last; ++i) {
            const int t = j.runs.tok[run.start + i];
            float v = 0.0f;
#pragma unroll
            for (int k = 0; k + 1 < TAPS; ++k) win[k] = win[k + 1];
            win[TAPS - 1] = j.in[(size_t)t * j.ld + c];
#pragma unroll
            for (int k = 0; k < TAPS; ++k) v += tap[k] * win[k];
            j.out[(size_t)t * C + c] = silu_f(v + bias);
        }
    } else {
        for (int i = first; i < last; ++i) {
            float v = 0.0f;
            for (int k = 0; k < K; ++k) v += w[k] * input(i - (K - 1) + k);
            j.out[(size_t)j.runs.tok[run.start + i] * C + c] = silu_f(v + bias);
        }
    }
    if (last == run.n)
        for (int k = 0; k < K - 1; ++k) new_in[(size_t)k * C + c] = input(run.n - (K - 1) + k);
}

}  // namespace

void short_conv(hipStream_t s, const ShortConv & j) {
    if (j.runs.n <= 0 || j.channels <= 0 || j.runs.longest <= 0) return;
    const dim3 grid((unsigned)((j.runs.longest + kConvTokens - 1) / kConvTokens), (unsigned)((j.channels + 255) / 256), (unsigned)j.runs.n);
    switch (j.taps) {
        case 2: hipLaunchKernelGGL(k_short_conv<2>, grid, dim3(256), 0, s, j); break;
        case 3: hipLaunchKernelGGL(k_short_conv<3>, grid, dim3(256), 0, s, j); break;
        case 4: hipLaunchKernelGGL(k_short_conv<4>, grid, dim3(256), 0, s, j); break;
        default: hipLaunchKernelGGL(k_short_conv<0>, grid, dim3(256), 0, s, j);
    }
    check_launch("short_conv");
}

}  // namespace rk
