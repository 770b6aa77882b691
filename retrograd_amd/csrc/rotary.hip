// Cosines and sines of a step's tokens for one set of rotary frequencies; layers that share the set share the table.
#include "stack_dev.hpp"

namespace rk {

namespace {

__global__ void k_rotary_table(const double * __restrict__ freq, int pairs, double magnitude, const int32_t * __restrict__ pos,
                               int n, float2 * __restrict__ table) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const int t = i / pairs;
    double s, c;
    sincos((double)pos[t] * freq[i - t * pairs], &s, &c);
    table[i] = make_float2((float)(c * magnitude), (float)(s * magnitude));
}

}  // namespace

void rotary_table(hipStream_t s, const double * freq, int pairs, double magnitude, const int32_t * pos, int T, float * table) {
    const int n = T * pairs;
    if (n <= 0) return;
    hipLaunchKernelGGL(k_rotary_table, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, freq, pairs, magnitude, pos, n, (float2 *)table);
    check_launch("rotary_table");
}

}  // namespace rk
