// The Mamba-2 mixer between its two projections: short causal convolution with SiLU over x, B and C (short_conv.hip), the
// state-space recurrence per head, and the gated grouped RMS norm. Everything here is f32 in both arithmetics; only the rows that
// leave for the output projection take the arithmetic's activation type.
#include "stack_dev.hpp"

namespace rk {

namespace {

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
    const SeqRun run = j.runs.runs[blockIdx.z];
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
            const float * row = j.xbc + (size_t)j.runs.tok[run.start + base + tk] * C + sh.inner() + g * N + n;
            sB[i] = row[0];
            sC[i] = row[(size_t)sh.groups * N];
        }
        if ((int)threadIdx.x < cnt) {
            const float dt = softplus_f(j.proj[(size_t)j.runs.tok[run.start + base + threadIdx.x] * j.ld + sh.inner() + C + h] + bias);
            s_dt[threadIdx.x] = dt;
            s_decay[threadIdx.x] = expf(-a * dt);
        }
        __syncthreads();
        for (int tk = 0; tk < cnt; ++tk) {
            const float x = mine ? j.xbc[(size_t)j.runs.tok[run.start + base + tk] * C + h * P + p] : 0.0f;
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
            const int t = j.runs.tok[run.start + base + tk];
            j.y[(size_t)t * sh.inner() + h * P + p] = y + D * j.xbc[(size_t)t * C + h * P + p];
        }
    }
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = q + 4 * i;
        if (mine && n < N) st[(size_t)n * P] = S[i];
    }
}

constexpr int kChunk = 64;            // tokens of a chunk
constexpr int kChunkP = 32;           // state columns of a workgroup
constexpr int kChunkN = 128;          // most state rows of the chunked kernel

// The recurrence in chunks of 64 tokens on the f32 matrix instruction. With l_t the running sum of -exp(A_log) dt in a
// chunk (kept in double: differences of it are what is exponentiated) and S the state before the chunk,
//   y_t = exp(l_t) S^T C_t + sum over s <= t of exp(l_t - l_s) dt_s (C_t . B_s) x_s + D x_t,
//   S  <- exp(l_last) S + sum over s of exp(l_last - l_s) dt_s B_s x_s^T.
// One workgroup walks a run's chunks for 32 columns of one head; wave w owns the chunk's token tile w. Tokens past the
// run's end count as dt = 0, which leaves everything unchanged. VEC: rows can be read four columns at a time, and the next
// chunk's rows are on their way while a chunk is worked on.
template <bool VEC>
__global__ __launch_bounds__(256) void k_mamba_chunks(MambaJob j) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const MambaShape sh = j.sh;
    const int N = sh.state, Np = (N + 15) / 16 * 16, P = sh.vdim, C = sh.channels(), LB = Np + 4;
    const int h = blockIdx.x, g = h / (sh.heads / sh.groups), p0 = blockIdx.y * kChunkP;
    const SeqRun run = j.runs.runs[blockIdx.z];
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, kg = lane >> 4;
    float * sB = sm, * sC = sB + kChunk * LB, * sX = sC + kChunk * LB, * sM = sX + kChunk * 36, * sS = sM + kChunk * 68;
    __shared__ double s_l[kChunk];
    __shared__ float s_dt[kChunk], s_w[kChunk];
    __shared__ int s_tok[kChunk];
    const float a = expf(j.A_log[h]), Dh = j.D[h], bias = j.dt_bias[h];
    float * st = j.state + (((size_t)run.slot * sh.heads + h) * N) * P + p0;
    const int n_tiles = Np / 16;
    // the state in registers: wave w holds row tiles w, w + 4, both column tiles
    f4 S[kChunkN / 64][2];
#pragma unroll
    for (int q = 0; q < kChunkN / 64; ++q)
#pragma unroll
        for (int c = 0; c < 2; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = (w + 4 * q) * 16 + 4 * kg + i, p = c * 16 + r16;
                S[q][c][i] = (n < N && p0 + p < P && !(run.flags & 1)) ? st[(size_t)n * P + p] : 0.0f;
            }
    constexpr int RB = kChunk * kChunkN / 4 / 256, RX = kChunk * kChunkP / 4 / 256;
    f4 nB[VEC ? RB : 1], nC[VEC ? RB : 1], nX[VEC ? RX : 1];
    float n_dt = 0.0f;
    int n_tok = 0;
    auto token = [&](int base, int tk) { return j.runs.tok[run.start + min(base + tk, run.n - 1)]; };
    auto fetch = [&](int base) {                // of the chunk at base into registers; nothing past the run's end is used
        if (w == 0) {
            n_tok = token(base, lane);
            n_dt = j.proj[(size_t)n_tok * j.ld + sh.inner() + C + h];
        }
        if constexpr (VEC) {
            const int n = 4 * (threadIdx.x & 31);
#pragma unroll
            for (int i = 0; i < RB; ++i) {
                const float * row = j.xbc + (size_t)token(base, (threadIdx.x >> 5) + 8 * i) * C + sh.inner() + g * N + min(n, N - 4);
                nB[i] = *(const f4 *)row;
                nC[i] = *(const f4 *)(row + (size_t)sh.groups * N);
            }
            const int p = 4 * (threadIdx.x & 7);
#pragma unroll
            for (int i = 0; i < RX; ++i)
                nX[i] = *(const f4 *)(j.xbc + (size_t)token(base, (threadIdx.x >> 3) + 32 * i) * C + h * P + min(p0 + p, P - 4));
        }
    };
    fetch(0);
    for (int base = 0; base < run.n; base += kChunk) {
        const int cnt = min(kChunk, run.n - base);
        __syncthreads();
        if (w == 0) {
            s_tok[lane] = n_tok;
            const float dt = lane < cnt ? softplus_f(n_dt + bias) : 0.0f;
            double l = -(double)a * (double)dt;
#pragma unroll
            for (int o = 1; o < 64; o <<= 1) {
                const double up = __shfl_up(l, o, 64);
                if (lane >= o) l += up;
            }
            s_l[lane] = l;
            s_dt[lane] = dt;
            s_w[lane] = expf((float)(__shfl(l, 63, 64) - l)) * dt;
        }
#pragma unroll
        for (int q = 0; q < kChunkN / 64; ++q)
#pragma unroll
            for (int c = 0; c < 2; ++c)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int n = (w + 4 * q) * 16 + 4 * kg + i;
                    if (n < Np) sS[n * 36 + c * 16 + r16] = S[q][c][i];
                }
        if constexpr (VEC) {
            const f4 zero = {0, 0, 0, 0};
            const int n = 4 * (threadIdx.x & 31), p = 4 * (threadIdx.x & 7);
            if (n < Np) {
#pragma unroll
                for (int i = 0; i < RB; ++i) {
                    const int tk = (threadIdx.x >> 5) + 8 * i;
                    const bool in = n < N && tk < cnt;
                    *(f4 *)(sB + tk * LB + n) = in ? nB[i] : zero;
                    *(f4 *)(sC + tk * LB + n) = in ? nC[i] : zero;
                }
            }
#pragma unroll
            for (int i = 0; i < RX; ++i) {
                const int tk = (threadIdx.x >> 3) + 32 * i;
                *(f4 *)(sX + tk * 36 + p) = p0 + p < P && tk < cnt ? nX[i] : zero;
            }
        } else {
            __syncthreads();
            for (int i = threadIdx.x; i < kChunk * Np; i += 256) {
                const int tk = i / Np, n = i - tk * Np;
                const float * row = j.xbc + (size_t)s_tok[tk] * C + sh.inner() + g * N + n;
                const bool in = n < N && tk < cnt;
                sB[tk * LB + n] = in ? row[0] : 0.0f;
                sC[tk * LB + n] = in ? row[(size_t)sh.groups * N] : 0.0f;
            }
            for (int i = threadIdx.x; i < kChunk * kChunkP; i += 256) {
                const int tk = i / kChunkP, p = i - tk * kChunkP;
                sX[tk * 36 + p] = (p0 + p < P && tk < cnt) ? j.xbc[(size_t)s_tok[tk] * C + h * P + p0 + p] : 0.0f;
            }
        }
        __syncthreads();
        if (base + kChunk < run.n) fetch(base + kChunk);
        const int t0 = 16 * w;
        double lt[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) lt[i] = s_l[t0 + 4 * kg + i];
        // decayed C B^T of this wave's tokens with everything before them
        for (int q = 0; q <= w; ++q) {
            f4 d = {0, 0, 0, 0};
            const float * ca = sC + (t0 + r16) * LB + 4 * kg, * cb = sB + (16 * q + r16) * LB + 4 * kg;
            for (int k = 0; k < Np; k += 16) {
                const f4 x = *(const f4 *)(ca + k), y = *(const f4 *)(cb + k);
#pragma unroll
                for (int e = 0; e < 4; ++e) d = __builtin_amdgcn_mfma_f32_16x16x4f32(x[e], y[e], d, 0, 0, 0);
            }
            const int sk = 16 * q + r16;
            const double ls = s_l[sk];
            const float dt = s_dt[sk];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = t0 + 4 * kg + i;
                sM[t * 68 + sk] = sk <= t ? d[i] * expf((float)(lt[i] - ls)) * dt : 0.0f;
            }
        }
        // (a wave reads only the rows of sM that it wrote)
        f4 y[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
        {
            const float * ca = sC + (t0 + r16) * LB + 4 * kg;
            for (int k = 0; k < Np; k += 16) {
                const f4 x = *(const f4 *)(ca + k);
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int c = 0; c < 2; ++c)
                        y[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(x[e], sS[(k + 4 * kg + e) * 36 + c * 16 + r16], y[c], 0, 0, 0);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float f = expf((float)lt[i]);
                y[0][i] *= f;
                y[1][i] *= f;
            }
            __builtin_amdgcn_wave_barrier();
            const float * ma = sM + (t0 + r16) * 68 + 4 * kg;
            for (int k = 0; k < t0 + 16; k += 16) {
                const f4 x = *(const f4 *)(ma + k);
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int c = 0; c < 2; ++c)
                        y[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(x[e], sX[(k + 4 * kg + e) * 36 + c * 16 + r16], y[c], 0, 0, 0);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int tk = t0 + 4 * kg + i;
            if (tk >= cnt) break;
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                const int p = c * 16 + r16;
                if (p0 + p < P) j.y[(size_t)s_tok[tk] * sh.inner() + h * P + p0 + p] = y[c][i] + Dh * sX[tk * 36 + p];
            }
        }
        const float decay = expf((float)s_l[kChunk - 1]);
#pragma unroll
        for (int q = 0; q < kChunkN / 64; ++q) {
            if (w + 4 * q >= n_tiles) break;
            f4 d[2] = {S[q][0] * decay, S[q][1] * decay};
            const int n = (w + 4 * q) * 16 + r16;
            for (int k = 0; k < cnt; k += 4) {
                const int sk = k + kg;
                const float bw = sB[sk * LB + n] * s_w[sk];
#pragma unroll
                for (int c = 0; c < 2; ++c) d[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(bw, sX[sk * 36 + c * 16 + r16], d[c], 0, 0, 0);
            }
            S[q][0] = d[0];
            S[q][1] = d[1];
        }
    }
#pragma unroll
    for (int q = 0; q < kChunkN / 64; ++q)
#pragma unroll
        for (int c = 0; c < 2; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = (w + 4 * q) * 16 + 4 * kg + i, p = c * 16 + r16;
                if (n < N && p0 + p < P) st[(size_t)n * P + p] = S[q][c][i];
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

void mamba_mix(hipStream_t s, int arith, const MambaJob & j, int T) {
    if (j.runs.n <= 0 || T <= 0) return;
    const MambaShape & sh = j.sh;
    if (sh.state > 512) throw std::runtime_error("mamba2: at most 512 state rows per head");
    ShortConv conv;
    conv.runs = j.runs;
    conv.channels = sh.channels(); conv.taps = sh.taps;
    conv.in = j.proj + sh.inner(); conv.ld = j.ld;
    conv.w = j.conv_w; conv.b = j.conv_b;
    conv.state = j.conv_state; conv.plane = j.conv_plane;
    conv.out = j.xbc;
    short_conv(s, conv);
    if (j.runs.longest >= kChunk / 2 && sh.state <= kChunkN) {
        const int Np = (sh.state + 15) / 16 * 16;
        const size_t lds = ((size_t)2 * kChunk * (Np + 4) + kChunk * 36 + kChunk * 68 + (size_t)Np * 36) * 4;
        constexpr int most = (2 * kChunk * (kChunkN + 4) + kChunk * 36 + kChunk * 68 + kChunkN * 36) * 4;
        static const bool allowed = hipFuncSetAttribute((const void *)k_mamba_chunks<true>, hipFuncAttributeMaxDynamicSharedMemorySize, most) == hipSuccess
                                 && hipFuncSetAttribute((const void *)k_mamba_chunks<false>, hipFuncAttributeMaxDynamicSharedMemorySize, most) == hipSuccess;
        if (!allowed) throw std::runtime_error("mamba2: a chunk does not fit the LDS");
        const dim3 grid((unsigned)sh.heads, (unsigned)((sh.vdim + kChunkP - 1) / kChunkP), (unsigned)j.runs.n);
        // every row starts at a multiple of four floats
        if (sh.vdim % 4 == 0 && sh.state % 4 == 0) hipLaunchKernelGGL(k_mamba_chunks<true>, grid, dim3(256), lds, s, j);
        else hipLaunchKernelGGL(k_mamba_chunks<false>, grid, dim3(256), lds, s, j);
        check_launch("mamba_chunks");
    } else {
        const dim3 grid((unsigned)sh.heads, (unsigned)((sh.vdim + kScanP - 1) / kScanP), (unsigned)j.runs.n);
        const size_t lds = (size_t)(2 * kScanTokens * sh.state + kScanTokens * 256) * 4;
        const int npt = (sh.state + 3) / 4;
        if (npt <= 8) hipLaunchKernelGGL(k_mamba_scan<8>, grid, dim3(256), lds, s, j);
        else if (npt <= 16) hipLaunchKernelGGL(k_mamba_scan<16>, grid, dim3(256), lds, s, j);
        else if (npt <= 32) hipLaunchKernelGGL(k_mamba_scan<32>, grid, dim3(256), lds, s, j);
        else if (npt <= 64) hipLaunchKernelGGL(k_mamba_scan<64>, grid, dim3(256), lds, s, j);
        else hipLaunchKernelGGL(k_mamba_scan<128>, grid, dim3(256), lds, s, j);
        check_launch("mamba_scan");
    }
    const dim3 gn((unsigned)T, (unsigned)sh.norm_groups);
    const size_t nl = (size_t)(sh.inner() / sh.norm_groups) * 4;
    if (arith == ARITH_16) hipLaunchKernelGGL(k_mamba_gate_norm<ARITH_16>, gn, dim3(256), nl, s, j);
    else hipLaunchKernelGGL(k_mamba_gate_norm<ARITH_32>, gn, dim3(256), nl, s, j);
    check_launch("mamba_gate_norm");
}

}  // namespace rk
