// Recurrent mixers with a matrix state - the gated delta rule with a decay per key channel or per head, and linear attention with
// a forget gate - between their projections (stack_kernels.hpp: DeltaJob). Everything here is f32 in both arithmetics; only the rows that leave for the output projection take the arithmetic's activation type.
// Short runs (decoding above all) take one launch from the projections' rows to those activations: a workgroup per run and
// head convolves its channels, walks the tokens with the state in registers and norms and gates the read-outs. Long runs are
// worked on in chunks of 64 tokens: everything inside a chunk that does not need the state, for all chunks at once; then the
// chunks one after the other with the state; then the read-outs.
#include "stack_dev.hpp"

#include <climits>
#include <type_traits>

namespace rk {

namespace {

constexpr int kChunk = 64;            // tokens of a chunk
constexpr int kLongRun = 32;          // tokens from which a run is worked on in chunks
constexpr int kChunkD = 128;          // most key channels of the chunk kernels
constexpr int kScanRows = 16;         // most rows of the state a thread of the scan holds

int pad16(int n) { return (n + 15) / 16 * 16; }

// c: the head's channel, or the head where it has one decay.
__device__ __forceinline__ float log_decay(const DeltaJob & j, int t, int c, float rate) {
    return -rate * softplus_f(j.decay[(size_t)t * j.ld_low + c] + j.dt_bias[c]);
}

// The forget gate of a channel: g = lower + (1 - lower) sigmoid(z), and 1 - g, each without cancellation.
struct Forget {
    float keep, write;
    __device__ __forceinline__ Forget(float z, float lower) : keep(lower + (1.0f - lower) * sigmoid_f(z)), write((1.0f - lower) * sigmoid_f(-z)) {}
    __device__ __forceinline__ float log_keep() const { return write < 0.5f ? log1pf(-write) : logf(fmaxf(keep, 1e-37f)); }
};

// Eight columns c .. c + 7 of a head's read-out o, of which the first `left` are real.
template <int ARITH>
__device__ __forceinline__ void store_read_out(const DeltaJob & j, int t, int h, int c, int left, const float (&o)[8], float inv) {
    const int col = h * j.sh.vdim + c;
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = i < left ? o[i] * inv * j.norm_w[c + i] : 0.0f;
    if (j.sh.gate != GATE_NONE) {
        const float * gate = j.gate + (size_t)t * j.ld_low + col;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const float z = i < left ? gate[i] : 0.0f, s = sigmoid_f(z);
            v[i] *= j.sh.gate == GATE_SILU ? z * s : s;
        }
    }
    if (left >= 8 && col % 8 == 0) {
        store_frag8<ARITH>(j.out, j.out_kf, t, col, v);
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            if (i >= left) break;
            const size_t at = frag_at(t, col + i, j.out_kf);
            if constexpr (ARITH == ARITH_16) ((uint16_t *)j.out)[at] = bf16_bits(v[i]);
            else ((float *)j.out)[at] = v[i];
        }
    }
}

// Runs of fewer than `below` tokens. Thread (rg, cg) holds rows rg, rg + RG, ... of four columns of the state; wider heads
// take several blocks of columns per token. The decayed state is multiplied with k and q in one pass: with u = beta (v - S^T k)
// the read-out after the write is S^T q + (k . q) u (forget rule: u = v).
template <int ARITH, int CG, int NPT>
__global__ __launch_bounds__(256) void k_delta_scan(DeltaJob j, int below) {
    constexpr int RG = 256 / CG;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ f4 red[2][4][2][CG];
    __shared__ float s_stat[4];
    const DeltaShape sh = j.sh;
    const SeqRun run = j.runs.runs[blockIdx.y];
    if (run.n >= below) return;
    const int D = sh.dim, V = sh.vdim, VP = sh.vpitch(), C = sh.channels(), K = sh.taps, KC = sh.keys();
    const int h = blockIdx.x, per = sh.heads / sh.kv_heads, kv = h / per;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, cg = tid % CG, rg = tid / CG;
    float * sv = sm, * so = sv + VP, * sq = so + VP, * sk = sq + D, * sg = sk + D;      // the columns first: whole groups of four
    const bool fresh = run.flags & 1;
    const int plane = (run.flags >> 1) & 1;
    const float * old_in = j.conv_state + (size_t)plane * j.conv_plane + (size_t)run.slot * (K - 1) * C;
    float * new_in = j.conv_state + (size_t)(1 - plane) * j.conv_plane + (size_t)run.slot * (K - 1) * C;
    float * st = j.state + ((size_t)run.slot * sh.heads + h) * (size_t)D * VP;
    const int n_blocks = (VP + 4 * CG - 1) / (4 * CG);
    f4 S[NPT];
    auto load_state = [&](int cb, bool zero) {
        const int c = cb * 4 * CG + 4 * cg;
#pragma unroll
        for (int i = 0; i < NPT; ++i) {
            const int n = rg + RG * i;
            S[i] = n < D && c < VP && !zero ? *(const f4 *)(st + (size_t)n * VP + c) : f4{0, 0, 0, 0};
        }
    };
    load_state(0, fresh);
    auto input = [&](int i, int c) -> float {          // input of the run's token i; i < 0: what the slot remembers
        if (i >= 0) return j.proj[(size_t)j.runs.tok[run.start + i] * j.ld + c];
        return fresh ? 0.0f : old_in[(size_t)(i + K - 1) * C + c];
    };
    auto channel = [&](int i) { return i < D ? kv * D + i : i < 2 * D ? KC + kv * D + i - D : 2 * KC + h * V + i - 2 * D; };
    const bool forget = sh.rule == RULE_FORGET;
    const float rate = forget ? 0.0f : expf(j.A_log[h]);
    if (tid < VP - V) sv[V + tid] = 0.0f;
    int parity = 0;
    for (int i = 0; i < run.n; ++i) {
        const int t = j.runs.tok[run.start + i];
        if (forget) {
            const float * row = j.proj + (size_t)t * j.ld;
            for (int d = tid; d < D; d += 256) {
                const Forget f(row[KC + h * D + d], j.lower[h * D + d]);
                sq[d] = silu_f(row[h * D + d]);
                sk[d] = f.write;
                sg[d] = f.keep;
            }
            for (int c = tid; c < V; c += 256) sv[c] = row[2 * KC + h * V + c];
        } else {
            for (int a = tid; a < 2 * D + V; a += 256) {
                const int c = channel(a);
                float x = 0.0f;
                for (int k = 0; k < K; ++k) x += j.conv_w[(size_t)c * K + k] * input(i - (K - 1) + k, c);
                x = silu_f(x);
                (a < D ? sq[a] : a < 2 * D ? sk[a - D] : sv[a - 2 * D]) = x;
            }
            for (int d = tid; d < D; d += 256) sg[d] = expf(log_decay(j, t, sh.rule == RULE_DELTA_HEADS ? h : h * D + d, rate));
        }
        __syncthreads();
        if (wave < 3) {                                 // the squares of q and k, and their product
            const float * a = wave == 1 ? sk : sq, * b = wave == 0 ? sq : sk;
            float x = 0.0f;
            for (int d = lane; d < D; d += 64) x += a[d] * b[d];
            x = wave_sum(x);
            if (lane == 0) s_stat[wave] = x;
        } else if (lane == 0 && !forget) {
            s_stat[3] = sigmoid_f(j.proj[(size_t)t * j.ld + C + h]);
        }
        __syncthreads();
        const float inv_q = forget ? 1.0f : 1.0f / sqrtf((s_stat[0] + j.unit_eps) * (float)D), inv_k = forget ? 1.0f : 1.0f / sqrtf(s_stat[1] + j.unit_eps);
        const float kq = s_stat[2] * inv_q * inv_k, beta = s_stat[3];
        for (int cb = 0; cb < n_blocks; ++cb) {
            const int c = cb * 4 * CG + 4 * cg;
            if (n_blocks > 1 && (i > 0 || cb > 0)) load_state(cb, fresh && i == 0);
            f4 held = {0, 0, 0, 0}, read = {0, 0, 0, 0};
#pragma unroll
            for (int r = 0; r < NPT; ++r) {
                const int n = rg + RG * r;
                if (n < D) {
                    S[r] *= sg[n];
                    held += S[r] * sk[n];
                    read += S[r] * sq[n];
                }
            }
#pragma unroll
            for (int o = CG; o < 64; o <<= 1)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    held[e] += __shfl_xor(held[e], o, 64);
                    read[e] += __shfl_xor(read[e], o, 64);
                }
            if (lane < CG) {
                red[parity][wave][0][cg] = held;
                red[parity][wave][1][cg] = read;
            }
            __syncthreads();
            held = red[parity][0][0][cg] + red[parity][1][0][cg] + red[parity][2][0][cg] + red[parity][3][0][cg];
            read = red[parity][0][1][cg] + red[parity][1][1][cg] + red[parity][2][1][cg] + red[parity][3][1][cg];
            parity ^= 1;
            f4 u = {0, 0, 0, 0};
            if (c < VP) u = forget ? *(const f4 *)(sv + c) : beta * (*(const f4 *)(sv + c) - held * inv_k);
            if (rg == 0 && c < VP) *(f4 *)(so + c) = read * inv_q + kq * u;
            const f4 w = u * inv_k;
#pragma unroll
            for (int r = 0; r < NPT; ++r) {
                const int n = rg + RG * r;
                if (n < D) S[r] += sk[n] * w;
            }
            if (c < VP && (n_blocks > 1 || i + 1 == run.n)) {
#pragma unroll
                for (int r = 0; r < NPT; ++r) {
                    const int n = rg + RG * r;
                    if (n < D) *(f4 *)(st + (size_t)n * VP + c) = S[r];
                }
            }
        }
        __syncthreads();
        float x = 0.0f;
        for (int c = lane; c < V; c += 64) x += so[c] * so[c];
        const float inv = 1.0f / sqrtf(wave_sum(x) / (float)V + j.eps);
        for (int c = 8 * tid; c < V; c += 8 * 256) {
            float o[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = c + e < V ? so[c + e] : 0.0f;
            store_read_out<ARITH>(j, t, h, c, V - c, o, inv);
        }
    }
    for (int a = tid; a < 2 * D + V; a += 256) {
        if (a < 2 * D && h % per != 0) continue;        // heads that share their keys: one leaves the inputs
        const int c = channel(a);
        for (int k = 0; k < K - 1; ++k) new_in[(size_t)k * C + c] = input(run.n - (K - 1) + k, c);
    }
}

// Scratch of the chunk kernels. Row p of a head belongs to place p of the step's tokens in run order.
struct Chunks {
    float * w, * q, * k, * u, * a, * last;
    int T, Dp, Vp, n_last;
    __device__ __forceinline__ size_t row(int h, int p) const { return (size_t)h * T + p; }
    __device__ __forceinline__ float * last_of(int h, int run, int start, int chunk) const { return last + ((size_t)h * n_last + start / kChunk + run + chunk) * Dp; }
};

// Running sums over the 16 lanes of a row.
__device__ __forceinline__ float row_scan(float v) {
    auto up = [](float x, auto n) { return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), 0x110 + decltype(n)::value, 0xf, 0xf, true)); };
    v += up(v, std::integral_constant<int, 1>());
    v += up(v, std::integral_constant<int, 2>());
    v += up(v, std::integral_constant<int, 4>());
    v += up(v, std::integral_constant<int, 8>());
    return v;
}

// What a chunk does to any state it may start from. With l_t the sum of the log decays up to token t of the chunk (per
// channel) and L[t][s] = beta_t sum_d k_t[d] k_s[d] exp(l_t - l_s)[d] for s < t, the written rows are
//   u = (1 + L)^-1 diag(beta) (v - (k exp(l)) S) = U - W S,
// and with A[t][s] = sum_d q_t[d] k_s[d] exp(l_t - l_s)[d] for s <= t
//   o = (q exp(l)) S + A u,   S' = exp(l_last) S + (k exp(l_last - l))^T u.
// One workgroup per chunk and head leaves W, U, A, q exp(l), k exp(l_last - l) and exp(l_last). Wave w owns the tokens of
// block w (16 of them), lane (r16, kg) of token r16 the channels 16 e + 4 kg .. + 3 - a matrix operand's layout. Decays are only ever
// exponentiated as sums over a stretch of tokens, so nothing grows: inside a block pair by pair, between blocks from the
// start of the one and to the end of the other. (1 + L)^-1 is applied by blocks of 16, whose own inverses are formed first.
// Tokens past the run's end count as k = q = beta = 0 without decay, which changes nothing.
// A decay per head comes out of the sums: products of k and q on the matrix instruction, then the factor of each pair, from sums in
// double since differences of them are exponentiated. Under the forget rule u is v, and there is no L, W or U.
template <int DT, int RULE> constexpr int chunk_lds_floats() {
    constexpr int Dp = 16 * DT, rows = kChunk * (Dp + 4), pairs = kChunk * (kChunk + 4);
    return rows + (RULE == RULE_DELTA_HEADS ? 0 : rows + 4 * Dp) + pairs + (RULE == RULE_FORGET ? 0 : pairs + kChunk * 20);
}
template <int DT, int RULE>
__global__ __launch_bounds__(256) void k_delta_chunk(DeltaJob j, Chunks out) {
    constexpr bool HEADS = RULE == RULE_DELTA_HEADS, FORGET = RULE == RULE_FORGET;
    constexpr int Dp = 16 * DT, LD = Dp + 4, LA = kChunk + 4;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const DeltaShape sh = j.sh;
    const SeqRun run = j.runs.runs[blockIdx.z];
    const int base = blockIdx.x * kChunk, h = blockIdx.y;
    if (run.n < kLongRun || base >= run.n) return;
    const int cnt = min(kChunk, run.n - base);
    const int D = sh.dim, V = sh.vdim, C = sh.channels(), KC = sh.keys(), kv = h / (sh.heads / sh.kv_heads);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, kg = lane >> 4;
    float * sK = sm, * sA = sK + kChunk * LD, * sP = sA + kChunk * LA, * sT = HEADS ? sP : sP + kChunk * LD;
    float * sL = HEADS ? sT : sT + 4 * Dp, * sInv = sL + kChunk * LA;
    __shared__ float s_beta[kChunk];
    __shared__ int s_tok[kChunk];
    const int me = 16 * w + r16;                       // this lane's token
    const bool in = me < cnt;
    const int t = j.runs.tok[run.start + base + min(me, cnt - 1)];
    const float beta = in && !FORGET ? sigmoid_f(j.proj[(size_t)t * j.ld + C + h]) : 0.0f;
    if (!FORGET && kg == 0) {
        s_beta[me] = beta;
        s_tok[me] = t;
    }
    // a decay per head: lane s of every wave has the sum up to token s
    double l_sum = 0.0;
    if constexpr (HEADS) {
        l_sum = lane < cnt ? (double)log_decay(j, j.runs.tok[run.start + base + lane], h, expf(j.A_log[h])) : 0.0;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const double up = __shfl_up(l_sum, o, 64);
            if (lane >= o) l_sum += up;
        }
    }
    f4 q[DT], k[DT], p[HEADS ? 1 : DT];
    if constexpr (FORGET) {
        const float * row = j.proj + (size_t)t * j.ld + h * D;
#pragma unroll
        for (int e = 0; e < DT; ++e)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = 16 * e + 4 * kg + i;
                const bool real = in && d < D;
                const Forget f(real ? row[KC + d] : 0.0f, real ? j.lower[h * D + d] : 1.0f);
                q[e][i] = real ? silu_f(row[d]) : 0.0f;
                k[e][i] = f.write;
                p[e][i] = real ? f.log_keep() : 0.0f;
            }
    } else {
        const float * row = j.qkv + (size_t)t * C + kv * D;
        const float rate = HEADS ? 0.0f : expf(j.A_log[h]);
        float qq = 0.0f, kk = 0.0f;
#pragma unroll
        for (int e = 0; e < DT; ++e)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = 16 * e + 4 * kg + i;
                const bool real = in && d < D;
                q[e][i] = real ? row[d] : 0.0f;
                k[e][i] = real ? row[KC + d] : 0.0f;
                if constexpr (!HEADS) p[e][i] = real ? log_decay(j, t, h * D + d, rate) : 0.0f;
                qq += q[e][i] * q[e][i];
                kk += k[e][i] * k[e][i];
            }
        qq += __shfl_xor(qq, 16, 64);
        qq += __shfl_xor(qq, 32, 64);
        kk += __shfl_xor(kk, 16, 64);
        kk += __shfl_xor(kk, 32, 64);
        const float fq = 1.0f / sqrtf((qq + j.unit_eps) * (float)D), fk = 1.0f / sqrtf(kk + j.unit_eps);
#pragma unroll
        for (int e = 0; e < DT; ++e) {
            q[e] *= fq;
            k[e] *= fk;
        }
    }
#pragma unroll
    for (int e = 0; e < DT; ++e) {
        *(f4 *)(sK + me * LD + 16 * e + 4 * kg) = k[e];
        if constexpr (!HEADS) {
#pragma unroll
            for (int i = 0; i < 4; ++i) p[e][i] = row_scan(p[e][i]);       // up to this token, from the start of the block
            *(f4 *)(sP + me * LD + 16 * e + 4 * kg) = p[e];
            if (r16 == 15) *(f4 *)(sT + w * Dp + 16 * e + 4 * kg) = p[e];
        }
    }
    __syncthreads();
    if constexpr (HEADS) {
        // the blocks up to this one
        for (int b = 0; b <= w; ++b) {
            f4 kk = {0, 0, 0, 0}, qk = {0, 0, 0, 0};
#pragma unroll
            for (int e = 0; e < DT; ++e) {
                const f4 x = *(const f4 *)(sK + (16 * b + r16) * LD + 16 * e + 4 * kg);
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    kk = __builtin_amdgcn_mfma_f32_16x16x4f32(k[e][i], x[i], kk, 0, 0, 0);
                    qk = __builtin_amdgcn_mfma_f32_16x16x4f32(q[e][i], x[i], qk, 0, 0, 0);
                }
            }
            const int s = 16 * b + r16;
            const double ls = __shfl(l_sum, s, 64);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = 16 * w + 4 * kg + i;
                const float f = expf(fminf((float)(__shfl(l_sum, r, 64) - ls), 0.0f));
                sL[r * LA + s] = s < r ? s_beta[r] * kk[i] * f : 0.0f;
                sA[r * LA + s] = s <= r ? qk[i] * f : 0.0f;
            }
        }
    } else {
        // the block with itself
#pragma unroll 1
        for (int s0 = 0; s0 < 16; s0 += 4) {
            float kk[4] = {0, 0, 0, 0}, qk[4] = {0, 0, 0, 0};
#pragma unroll
            for (int e = 0; e < DT; ++e)
#pragma unroll
                for (int s = 0; s < 4; ++s) {
                    const f4 ks = *(const f4 *)(sK + (16 * w + s0 + s) * LD + 16 * e + 4 * kg), ps = *(const f4 *)(sP + (16 * w + s0 + s) * LD + 16 * e + 4 * kg);
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const float x = ks[i] * __expf(fminf(p[e][i] - ps[i], 0.0f));       // later tokens are left out below
                        if constexpr (!FORGET) kk[s] += k[e][i] * x;
                        qk[s] += q[e][i] * x;
                    }
                }
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                if constexpr (!FORGET) {
                    kk[s] += __shfl_xor(kk[s], 16, 64);
                    kk[s] += __shfl_xor(kk[s], 32, 64);
                }
                qk[s] += __shfl_xor(qk[s], 16, 64);
                qk[s] += __shfl_xor(qk[s], 32, 64);
            }
            if (kg == 0) {
                const int s = s0;
                if constexpr (!FORGET) *(f4 *)(sL + me * LA + 16 * w + s) = f4{s < r16 ? beta * kk[0] : 0.0f, s + 1 < r16 ? beta * kk[1] : 0.0f, s + 2 < r16 ? beta * kk[2] : 0.0f, s + 3 < r16 ? beta * kk[3] : 0.0f};
                *(f4 *)(sA + me * LA + 16 * w + s) = f4{s <= r16 ? qk[0] : 0.0f, s + 1 <= r16 ? qk[1] : 0.0f, s + 2 <= r16 ? qk[2] : 0.0f, s + 3 <= r16 ? qk[3] : 0.0f};
            }
        }
    }
    __syncthreads();
    // the block's own inverse, column r16 per lane
    if constexpr (!FORGET) {
        float x[16];
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            float v = r == r16 ? 1.0f : 0.0f;
#pragma unroll
            for (int s4 = 0; s4 < r; s4 += 4) {
                const f4 l = *(const f4 *)(sL + (16 * w + r) * LA + 16 * w + s4);
#pragma unroll
                for (int s = 0; s < 4; ++s) if (s4 + s < r) v -= l[s] * x[s4 + s];
            }
            x[r] = v;
        }
        if (kg == 0)
#pragma unroll
            for (int r = 0; r < 16; ++r) sInv[(16 * w + r) * 20 + r16] = x[r];
    }
    // from the start of the chunk, to its end, and within the block; what other blocks need of this one
    const size_t at = out.row(h, run.start + base + me) * Dp;
    if constexpr (HEADS) {
        const double l = __shfl(l_sum, me, 64), end = __shfl(l_sum, 63, 64);
        const float from = expf((float)l), to = expf((float)(end - l)), all = expf((float)end);
#pragma unroll
        for (int e = 0; e < DT; ++e) {
            const int c = 16 * e + 4 * kg;
            *(f4 *)(sK + me * LD + c) = k[e] * (beta * from);
            if (in) {
                *(f4 *)(out.q + at + c) = q[e] * from;
                *(f4 *)(out.k + at + c) = k[e] * to;
            }
            if (w == 0 && r16 == 0) *(f4 *)(out.last_of(h, blockIdx.z, run.start, blockIdx.x) + c) = f4{all, all, all, all};
        }
        __syncthreads();
    } else {
#pragma unroll
        for (int e = 0; e < DT; ++e) {
            const int c = 16 * e + 4 * kg;
            f4 before = {0, 0, 0, 0}, after = {0, 0, 0, 0};
            for (int b = 0; b < w; ++b) before += *(const f4 *)(sT + b * Dp + c);
            for (int b = w + 1; b < 4; ++b) after += *(const f4 *)(sT + b * Dp + c);
            const f4 own = *(const f4 *)(sT + w * Dp + c);
            f4 ke, qe, kr, kl;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float from = __expf(p[e][i]), f = __expf(before[i]), r = __expf(own[i] - p[e][i]);
                ke[i] = beta * k[e][i] * from * f;
                qe[i] = q[e][i] * from * f;
                kr[i] = k[e][i] * r;
                kl[i] = kr[i] * __expf(after[i]);
                k[e][i] *= from;
                q[e][i] *= from;
            }
            if constexpr (!FORGET) *(f4 *)(sK + me * LD + c) = ke;
            *(f4 *)(sP + me * LD + c) = kr;
            if (in) {
                *(f4 *)(out.q + at + c) = qe;
                *(f4 *)(out.k + at + c) = kl;
            }
            if (w == 0 && r16 == 0) {
                f4 l;
#pragma unroll
                for (int i = 0; i < 4; ++i) l[i] = __expf(own[i] + after[i]);
                *(f4 *)(out.last_of(h, blockIdx.z, run.start, blockIdx.x) + c) = l;
            }
        }
        __syncthreads();
        // with the blocks before it
        for (int b = 0; b < w; ++b) {
            f4 kk = {0, 0, 0, 0}, qk = {0, 0, 0, 0};
#pragma unroll
            for (int e = 0; e < DT; ++e) {
                const int c = 16 * e + 4 * kg;
                f4 x = *(const f4 *)(sP + (16 * b + r16) * LD + c);
                if (b + 1 < w) {
                    f4 between = {0, 0, 0, 0};
                    for (int m = b + 1; m < w; ++m) between += *(const f4 *)(sT + m * Dp + c);
#pragma unroll
                    for (int i = 0; i < 4; ++i) x[i] *= __expf(between[i]);
                }
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    if constexpr (!FORGET) kk = __builtin_amdgcn_mfma_f32_16x16x4f32(k[e][i], x[i], kk, 0, 0, 0);
                    qk = __builtin_amdgcn_mfma_f32_16x16x4f32(q[e][i], x[i], qk, 0, 0, 0);
                }
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = 16 * w + 4 * kg + i;
                if constexpr (!FORGET) sL[r * LA + 16 * b + r16] = s_beta[r] * kk[i];
                sA[r * LA + 16 * b + r16] = qk[i];
            }
        }
        __syncthreads();
    }
    // W and U, a tile of 16 columns at a time: block i of the solution is T_ii (Y_i - sum over b < i of L_ib X_b); a product's
    // result (rows 4 kg + i in register i) is the next one's operand with its K in that order
    const int n_tiles = FORGET ? 0 : DT + out.Vp / 16;
    for (int n = w; n < n_tiles; n += 4) {
        f4 X[4];
        const int c = (n < DT ? n : n - DT) * 16 + r16;
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            f4 y;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = 16 * b + 4 * kg + i;
                if (n < DT) y[i] = sK[r * LD + c];
                else y[i] = r < cnt && c < V ? s_beta[r] * j.qkv[(size_t)s_tok[r] * C + 2 * KC + h * V + c] : 0.0f;
            }
#pragma unroll
            for (int m = 0; m < b; ++m) {
                const f4 l = *(const f4 *)(sL + (16 * b + r16) * LA + 16 * m + 4 * kg);
#pragma unroll
                for (int i = 0; i < 4; ++i) y = __builtin_amdgcn_mfma_f32_16x16x4f32(-l[i], X[m][i], y, 0, 0, 0);
            }
            const f4 inv = *(const f4 *)(sInv + (16 * b + r16) * 20 + 4 * kg);
            X[b] = f4{0, 0, 0, 0};
#pragma unroll
            for (int i = 0; i < 4; ++i) X[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(inv[i], y[i], X[b], 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = 16 * b + 4 * kg + i;
                if (r >= cnt) continue;
                const size_t row = out.row(h, run.start + base + r);
                if (n < DT) out.w[row * Dp + c] = X[b][i];
                else out.u[row * out.Vp + c] = X[b][i];
            }
        }
    }
    for (int i = threadIdx.x; i < kChunk * kChunk / 4; i += 256) {
        const int r = i / (kChunk / 4), c = i % (kChunk / 4) * 4;
        if (r < cnt && c <= (r | 15)) *(f4 *)(out.a + out.row(h, run.start + base + r) * kChunk + c) = *(const f4 *)(sA + r * LA + c);
    }
}

// The chunks of a run one after the other, for NC tiles of 16 columns of one head's state. Wave w owns token block w of a chunk
// and rows w, w + 4 (in tiles of 16) of the state. The rows of the next chunk are requested as soon as a chunk's were used.
// DELTA: u = U - W S; otherwise u = v, as projected.
template <int DT, bool DELTA, int NC>
__global__ __launch_bounds__(256) void k_delta_walk(DeltaJob j, Chunks in, int col_blocks) {
    constexpr int Dp = 16 * DT, NT = (DT + 3) / 4, LS = 16 * NC + 4;
    __shared__ __attribute__((aligned(16))) float sS[Dp * LS], sU[kChunk * LS];
    const DeltaShape sh = j.sh;
    const SeqRun run = j.runs.runs[blockIdx.y];
    if (run.n < kLongRun) return;
    // workgroup b runs on XCD b % 8: the column blocks of a head share its rows in one L2
    const int group = (blockIdx.x >> 3) / col_blocks * 8 + (blockIdx.x & 7), p0 = (blockIdx.x >> 3) % col_blocks * 16 * NC, h = group;
    if (h >= sh.heads) return;
    const int D = sh.dim, V = sh.vdim, VP = sh.vpitch();
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, kg = lane >> 4, t0 = 16 * w;
    float * st = j.state + ((size_t)run.slot * sh.heads + h) * (size_t)D * VP + p0;
    f4 S[NT][NC];
#pragma unroll
    for (int d = 0; d < NT; ++d)
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = (w + 4 * d) * 16 + 4 * kg + i, p = c * 16 + r16;
                S[d][c][i] = n < D && p0 + p < V && !(run.flags & 1) ? st[(size_t)n * VP + p] : 0.0f;
            }
    f4 rw[DELTA ? DT : 1], rq[DT], ra[4], ru[NC], rk[NT][4], rl[NT];
    int v_tok[4];                                // tokens of the lane's values in the chunk that is fetched next
    auto fetch_tokens = [&](int base) {
        if constexpr (!DELTA)
#pragma unroll
            for (int i = 0; i < 4; ++i) v_tok[i] = j.runs.tok[run.start + min(base + t0 + 4 * kg + i, run.n - 1)];
    };
    auto fetch_first = [&](int base) {          // what the first products of the chunk at base read
        const int cnt = min(kChunk, run.n - base);
        const bool mine = t0 + r16 < cnt;
        const size_t at = in.row(h, run.start + base + min(t0 + r16, cnt - 1)) * Dp + 4 * kg;
#pragma unroll
        for (int e = 0; e < DT; ++e) {
            if constexpr (DELTA) rw[e] = *(const f4 *)(in.w + at + 16 * e);
            rq[e] = *(const f4 *)(in.q + at + 16 * e);
        }
        if (!mine)
#pragma unroll
            for (int e = 0; e < DT; ++e) {
                rq[e] = f4{0, 0, 0, 0};
                if constexpr (DELTA) rw[e] = f4{0, 0, 0, 0};
            }
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = t0 + 4 * kg + i, p = p0 + c * 16 + r16;
                if constexpr (DELTA) ru[c][i] = r < cnt && p < in.Vp ? in.u[in.row(h, run.start + base + r) * in.Vp + p] : 0.0f;
                else ru[c][i] = r < cnt && p < V ? j.proj[(size_t)v_tok[i] * j.ld + 2 * sh.keys() + h * V + p] : 0.0f;
            }
        fetch_tokens(base + kChunk);
    };
    auto fetch_second = [&](int base) {
        const int cnt = min(kChunk, run.n - base);
        const bool mine = t0 + r16 < cnt;
        const size_t at = in.row(h, run.start + base + min(t0 + r16, cnt - 1)) * kChunk + 4 * kg;
#pragma unroll
        for (int q = 0; q < 4; ++q) ra[q] = q <= w && mine ? *(const f4 *)(in.a + at + 16 * q) : f4{0, 0, 0, 0};
        const float * last = in.last_of(h, blockIdx.y, run.start, base / kChunk);
#pragma unroll
        for (int d = 0; d < NT; ++d) {
            if (w + 4 * d >= DT) break;
            rl[d] = *(const f4 *)(last + (w + 4 * d) * 16 + 4 * kg);
#pragma unroll
            for (int q = 0; q < 4; ++q)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int r = 16 * q + 4 * kg + i;
                    rk[d][q][i] = r < cnt ? in.k[in.row(h, run.start + base + r) * Dp + (w + 4 * d) * 16 + r16] : 0.0f;
                }
        }
    };
    fetch_tokens(0);
    fetch_first(0);
    fetch_second(0);
    for (int base = 0; base < run.n; base += kChunk) {
        const int cnt = min(kChunk, run.n - base);
#pragma unroll
        for (int d = 0; d < NT; ++d) {
            if (w + 4 * d >= DT) break;
#pragma unroll
            for (int c = 0; c < NC; ++c)
#pragma unroll
                for (int i = 0; i < 4; ++i) sS[((w + 4 * d) * 16 + 4 * kg + i) * LS + c * 16 + r16] = S[d][c][i];
        }
        __syncthreads();
        f4 u[NC], o[NC];
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            u[c] = ru[c];
            o[c] = f4{0, 0, 0, 0};
        }
#pragma unroll
        for (int e = 0; e < DT; ++e)
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int c = 0; c < NC; ++c) {
                    const float s = sS[(16 * e + 4 * kg + i) * LS + c * 16 + r16];
                    if constexpr (DELTA) u[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(-rw[e][i], s, u[c], 0, 0, 0);
                    o[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(rq[e][i], s, o[c], 0, 0, 0);
                }
        if (base + kChunk < run.n) fetch_first(base + kChunk);
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) sU[(t0 + 4 * kg + i) * LS + c * 16 + r16] = u[c][i];
        __syncthreads();
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            if (q > w) break;
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int c = 0; c < NC; ++c) o[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(ra[q][i], sU[(16 * q + 4 * kg + i) * LS + c * 16 + r16], o[c], 0, 0, 0);
        }
#pragma unroll
        for (int d = 0; d < NT; ++d) {
            if (w + 4 * d >= DT) break;
#pragma unroll
            for (int c = 0; c < NC; ++c) S[d][c] *= rl[d];
#pragma unroll
            for (int q = 0; q < 4; ++q)
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int c = 0; c < NC; ++c)
                        S[d][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(rk[d][q][i], sU[(16 * q + 4 * kg + i) * LS + c * 16 + r16], S[d][c], 0, 0, 0);
        }
        if (base + kChunk < run.n) fetch_second(base + kChunk);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = t0 + 4 * kg + i;
            if (r >= cnt) break;
            const int t = j.runs.tok[run.start + base + r];
#pragma unroll
            for (int c = 0; c < NC; ++c) {
                const int p = p0 + c * 16 + r16;
                if (p < V) j.y[(size_t)t * sh.inner() + h * V + p] = o[c][i];
            }
        }
    }
#pragma unroll
    for (int d = 0; d < NT; ++d)
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int n = (w + 4 * d) * 16 + 4 * kg + i, p = c * 16 + r16;
                if (n < D && p0 + p < V) st[(size_t)n * VP + p] = S[d][c][i];
            }
}

// Norm and gate of the read-outs of long runs: `lanes` lanes per head, eight columns each.
template <int ARITH>
__global__ __launch_bounds__(256) void k_delta_read_out(DeltaJob j, int lanes) {
    const DeltaShape sh = j.sh;
    const SeqRun run = j.runs.runs[blockIdx.z];
    const int i = blockIdx.x, h = blockIdx.y * (256 / lanes) + threadIdx.x / lanes, sub = threadIdx.x % lanes;
    if (run.n < kLongRun || i >= run.n) return;
    const int t = j.runs.tok[run.start + i], V = sh.vdim;
    const bool real = h < sh.heads;
    const float * y = j.y + (size_t)t * sh.inner() + (real ? h : 0) * V;
    const bool even = V % 4 == 0;
    auto load = [&](int c, float (&o)[8]) {
        if (even && c + 8 <= V) {
            const f4 a = *(const f4 *)(y + c), b = *(const f4 *)(y + c + 4);
#pragma unroll
            for (int e = 0; e < 4; ++e) { o[e] = a[e]; o[4 + e] = b[e]; }
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = c + e < V ? y[c + e] : 0.0f;
        }
    };
    float q = 0.0f, o[8];
    for (int c = 8 * sub; c < V; c += 8 * lanes) {
        load(c, o);
#pragma unroll
        for (int e = 0; e < 8; ++e) q += o[e] * o[e];
    }
    for (int m = 1; m < lanes; m <<= 1) q += __shfl_xor(q, m, 64);
    if (!real) return;
    const float inv = 1.0f / sqrtf(q / (float)V + j.eps);
    for (int c = 8 * sub; c < V; c += 8 * lanes) {
        load(c, o);
        store_read_out<ARITH>(j, t, h, c, V - c, o, inv);
    }
}

bool in_chunks(const DeltaShape & sh) { return sh.dim <= kChunkD; }
// The compiled numbers of 16-channel tiles.
int chunk_tiles(int dim) {
    for (int n : {1, 2, 3, 4, 6, 8}) if (dim <= 16 * n) return n;
    return 0;
}

Chunks chunks_of(const DeltaShape & sh, int T, int n_runs, float * base) {
    Chunks c;
    c.T = T;
    c.Dp = 16 * chunk_tiles(sh.dim);
    c.Vp = pad16(sh.vdim);
    c.n_last = T / kChunk + n_runs + 1;
    const size_t rows = (size_t)sh.heads * T;
    c.w = base;
    c.q = c.w + rows * c.Dp;
    c.k = c.q + rows * c.Dp;
    c.u = c.k + rows * c.Dp;
    c.a = c.u + rows * c.Vp;
    c.last = c.a + rows * kChunk;
    return c;
}

template <int DT, int RULE> void launch_chunks(hipStream_t s, const DeltaJob & j, const Chunks & c) {
    const DeltaShape & sh = j.sh;
    constexpr int lds = chunk_lds_floats<DT, RULE>() * 4;
    static const bool allowed = hipFuncSetAttribute((const void *)k_delta_chunk<DT, RULE>, hipFuncAttributeMaxDynamicSharedMemorySize, lds) == hipSuccess;
    if (!allowed) throw std::runtime_error("matrix states: a chunk does not fit the LDS");
    const unsigned n_chunks = (unsigned)((j.runs.longest + kChunk - 1) / kChunk);
    hipLaunchKernelGGL((k_delta_chunk<DT, RULE>), dim3(n_chunks, (unsigned)sh.heads, (unsigned)j.runs.n), dim3(256), lds, s, j, c);
    check_launch("delta_chunk");
    // narrower blocks of columns while there are CUs for them: a chunk is a chain of products either way
    const bool narrow = (int64_t)sh.heads * ((sh.vdim + 31) / 32) * j.runs.n <= 128;
    const int blocks = narrow ? (sh.vdim + 15) / 16 : (sh.vdim + 31) / 32;
    const dim3 grid((unsigned)((sh.heads + 7) / 8 * 8 * blocks), (unsigned)j.runs.n);
    if (narrow) hipLaunchKernelGGL((k_delta_walk<DT, RULE != RULE_FORGET, 1>), grid, dim3(256), 0, s, j, c, blocks);
    else hipLaunchKernelGGL((k_delta_walk<DT, RULE != RULE_FORGET, 2>), grid, dim3(256), 0, s, j, c, blocks);
    check_launch("delta_walk");
}

template <int RULE> void launch_chunks(hipStream_t s, const DeltaJob & j, const Chunks & c) {
    switch (chunk_tiles(j.sh.dim)) {
        case 1: launch_chunks<1, RULE>(s, j, c); break;
        case 2: launch_chunks<2, RULE>(s, j, c); break;
        case 3: launch_chunks<3, RULE>(s, j, c); break;
        case 4: launch_chunks<4, RULE>(s, j, c); break;
        case 6: launch_chunks<6, RULE>(s, j, c); break;
        default: launch_chunks<8, RULE>(s, j, c); break;
    }
}

template <int ARITH, int CG, int NPT> void launch_scan(hipStream_t s, const DeltaJob & j, int below) {
    const DeltaShape & sh = j.sh;
    const size_t lds = (size_t)(2 * sh.vpitch() + 3 * sh.dim) * 4;
    hipLaunchKernelGGL((k_delta_scan<ARITH, CG, NPT>), dim3((unsigned)sh.heads, (unsigned)j.runs.n), dim3(256), lds, s, j, below);
    check_launch("delta_scan");
}
template <int ARITH, int CG> void launch_scan(hipStream_t s, const DeltaJob & j, int below) {
    const int npt = (j.sh.dim + 256 / CG - 1) / (256 / CG);
    if (npt <= 1) launch_scan<ARITH, CG, 1>(s, j, below);
    else if (npt <= 2) launch_scan<ARITH, CG, 2>(s, j, below);
    else if (npt <= 4) launch_scan<ARITH, CG, 4>(s, j, below);
    else if (npt <= 8) launch_scan<ARITH, CG, 8>(s, j, below);
    else launch_scan<ARITH, CG, kScanRows>(s, j, below);
}
template <int ARITH> void scan(hipStream_t s, const DeltaJob & j, int below) {
    // as many columns side by side as the head has, unless a thread then held too many rows
    const int d = j.sh.dim, v = j.sh.vdim;
    if (v > 64 && d <= 8 * kScanRows) launch_scan<ARITH, 32>(s, j, below);
    else if (v > 32 && d <= 16 * kScanRows) launch_scan<ARITH, 16>(s, j, below);
    else launch_scan<ARITH, 8>(s, j, below);
}

}  // namespace

size_t delta_chunk_floats(const DeltaShape & sh, int T, int n_runs) {
    if (!in_chunks(sh)) return 0;
    const Chunks c = chunks_of(sh, T, n_runs, nullptr);
    return (size_t)sh.heads * ((size_t)T * (3 * c.Dp + c.Vp + kChunk) + (size_t)c.n_last * c.Dp);
}

void delta_mix(hipStream_t s, int arith, const DeltaJob & j, int T) {
    if (j.runs.n <= 0 || T <= 0) return;
    const DeltaShape & sh = j.sh;
    if (sh.dim > 32 * kScanRows || sh.vdim > 4096) throw std::runtime_error("matrix states: at most 512 key and 4096 value channels per head");
    const int least = in_chunks(sh) ? kLongRun : INT_MAX;
    if (j.runs.longest >= least) {
        if (sh.rule != RULE_FORGET) {
            ShortConv conv;
            conv.runs = j.runs;
            conv.channels = sh.channels(); conv.taps = sh.taps; conv.least = least;
            conv.in = j.proj; conv.ld = j.ld;
            conv.w = j.conv_w;
            conv.state = j.conv_state; conv.plane = j.conv_plane;
            conv.out = j.qkv;
            short_conv(s, conv);
        }
        const Chunks c = chunks_of(sh, T, j.runs.n, j.chunks);
        switch (sh.rule) {
            case RULE_DELTA_CHANNELS: launch_chunks<RULE_DELTA_CHANNELS>(s, j, c); break;
            case RULE_DELTA_HEADS: launch_chunks<RULE_DELTA_HEADS>(s, j, c); break;
            default: launch_chunks<RULE_FORGET>(s, j, c); break;
        }
        int lanes = 1;
        while (lanes < 64 && 8 * lanes < sh.vdim) lanes *= 2;
        const dim3 grid((unsigned)j.runs.longest, (unsigned)((sh.heads * lanes + 255) / 256), (unsigned)j.runs.n);
        if (arith == ARITH_16) hipLaunchKernelGGL(k_delta_read_out<ARITH_16>, grid, dim3(256), 0, s, j, lanes);
        else hipLaunchKernelGGL(k_delta_read_out<ARITH_32>, grid, dim3(256), 0, s, j, lanes);
        check_launch("delta_read_out");
    }
    if (j.runs.shortest < least) {
        if (arith == ARITH_16) scan<ARITH_16>(s, j, least);
        else scan<ARITH_32>(s, j, least);
    }
}

}  // namespace rk
