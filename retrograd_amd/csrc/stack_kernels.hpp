// Launch interface of the kernels behind layer-stack models (safetensors checkpoints whose config lists every layer):
// bf16-weight matrix products in two arithmetics (also over the tokens of every expert), norms, rotary positions, paged
// attention, expert routing, the state-space mixer.
#pragma once

#include "kernels.hpp"

namespace rk {

// The two arithmetics of a layer-stack model. ARITH_16: matrix products and the activations between kernels in
// bfloat16 with f32 accumulation, the latent cache in f16. ARITH_32: everything in f32 (products on the f32 matrix
// instruction; the stored bf16 weights widen exactly).
enum : int { ARITH_16 = 2, ARITH_32 = 4 };       // the value is the bytes of an activation element

// ---- dense matrices and activations in operand ("fragment") order -------------------------------
// Rows (of a weight, or tokens of an activation buffer) in tiles of 16, columns in fragments of 32:
//   [row / 16][k / 32][lane = 16 * ((k % 32) / 8) + row % 16][k % 8]
// so that a wave's operand of a 16x16x32 product is one contiguous load. Padding rows and columns of weights are zero;
// padding columns of activations only have to be finite. Activation buffers hold a multiple of FRAG_ROWS tokens.
constexpr int FRAG_ROWS = 128;
constexpr int frags_of(int k) { return (k + 31) / 32; }
constexpr size_t frag_elems(int rows, int kf) { return (size_t)((rows + FRAG_ROWS - 1) / FRAG_ROWS) * FRAG_ROWS * (size_t)kf * 32; }
constexpr size_t frag_weight_elems(int row_tiles, int kf) { return (size_t)row_tiles * (size_t)kf * 512; }

// `batch` matrices of `tiles` row tiles (n true rows) and kf fragments, one behind the other, stored as bf16.
struct DenseWeight {
    const uint16_t * w = nullptr;
    int n = 0, tiles = 0, kf = 0, batch = 1;
    size_t bytes() const { return frag_weight_elems(tiles, kf) * 2 * (size_t)batch; }
};
// Places of consecutive rows or columns: `run` of them side by side, runs `step` apart.
struct PackMap {
    int at, run, step;
    PackMap(int at, int run = 1 << 30, int step = 1 << 30) : at(at), run(run), step(step) {}
};
// dst(row(r), column(k)) = src[r * row_stride + k * k_stride] for r < rows, k < cols; dst has kf fragments per row tile.
void dense_pack(hipStream_t s, const uint16_t * src, int rows, int cols, int64_t row_stride, int64_t k_stride,
                uint16_t * dst, int kf, PackMap row, PackMap column);

// Where a product's rows go. col0 + b * col_batch + n is the output column of row n of batch b.
enum : int {
    OUT_F32 = 0,        // f32 rows dst[t * ld + col] = scale * v
    OUT_ACT,            // activations in fragment order, ld fragments per token tile: scale * v
    OUT_ACT_RELU2,      // ... max(v, 0)^2
    OUT_ACT_GATED,      // ... v * sigmoid(gate[t * ld_gate + b])
    OUT_QUERY,          // rows [t][batch][ld] in the cache's element type (f16 or f32): scale * v
    OUT_RESIDUAL,       // f32 rows dst[t * ld + col] += v
    OUT_ACT_GEGLU,      // activations from pairs of row tiles (gate, then up): gelu(gate) * up, gelu in its tanh form
    OUT_ACT_SWIGLU,     // ... silu(gate) * up
    OUT_ROTARY,         // queries, keys and values of grouped attention (RotaryOut)
    OUT_EXPERT,         // f32 rows dst[choice * stride + token * ld + col] = weight * v of an expert product's pairs
    OUT_ACT_CLAMPED,    // ... g * sigmoid(slope * g) * (u + 1) of g = min(gate, limit), u = up clamped to [-limit, limit]
    OUT_F32_CAPPED,     // f32 rows dst[t * ld + col] = limit * tanh(v / limit)
};
constexpr bool out_is_glu(int kind) { return kind == OUT_ACT_GEGLU || kind == OUT_ACT_SWIGLU || kind == OUT_ACT_CLAMPED; }

// Rows of a product that are heads of kf * 32 columns, H of queries, then G of keys: rotated, the queries to rows
// [t][H][kf * 32], the keys to their cells. The values are the keys as projected (vf 0), or G heads of vf * 32 columns behind
// them. The columns of a rotated pair are neighbours (2 i, 2 i + 1).
struct RotaryOut {
    int H = 0, G = 0, kf = 0, vf = 0, pairs = 0;      // rotated pairs of a head
    const float * table = nullptr;             // [T][pairs][2]: cosine and sine
    void * k_pool = nullptr, * v_pool = nullptr;
    const int32_t * cell = nullptr;
};
struct DenseOut {
    int kind = OUT_F32;
    void * dst = nullptr;
    int ld = 0, col0 = 0, col_batch = 0;
    float scale = 1.0f;
    float limit = 0.0f, slope = 1.0f;          // of the clamped gated pair (its gate's sigmoid), of the soft cap
    const float * gate = nullptr;
    int ld_gate = 0;
    size_t stride = 0;
    RotaryOut rot;
};
struct DenseIn {
    const void * x = nullptr;   // activations in fragment order
    int kf = 0;                 // fragments per token tile of that buffer
    int kf_batch = 0;           // batch b reads from fragment b * kf_batch on
};
// One product, or two with one weight buffer [first | second] along K whose results are scaled element by element and
// added: v = scale1[n] * (W1 x1) + scale2[n] * (W2 x2) (kf1 fragments belong to the first; scale1 null: plain product).
// With token_gate, v is multiplied by sigmoid(token_gate[t * ld_token_gate]) (OUT_RESIDUAL).
// With groups, batch b of the weight multiplies the pairs (token, choice) that chose expert b: their slots are the
// product's columns, read as tokens (gather; x then holds plain rows of kf * 32 columns, so that a gathered row's pieces
// lie together) or as rows of a buffer in slot order.
struct ExpertGroups {
    const int32_t * tiles = nullptr;           // [max_tiles][4]: expert, first slot (a multiple of 16), slots
    const int32_t * n_tiles = nullptr;
    int max_tiles = 0, block = 0;              // most slots of a tile: expert_block()
    const int32_t * slot_pair = nullptr;       // the pair of a slot
    const float * weight = nullptr;            // of a pair
    int top = 0, pairs = 0;
    bool weigh_input = false;                  // a pair's weight multiplies what its expert reads, not what it leaves
};
struct DenseJob {
    DenseWeight w;
    DenseIn x, x2;
    int kf1 = 0;
    const float * scale1 = nullptr, * scale2 = nullptr;
    int split_tile = 0;         // row tiles below go to `a`, the others (their rows counted from there) to `b`
    DenseOut a, b;
    int n_a = 0;                // true rows of part a when there is a part b
    const float * token_gate = nullptr;
    int ld_token_gate = 0;
    const float * bias = nullptr;              // [batch][tiles * 16], in the weight's row order, added to the product
    const ExpertGroups * groups = nullptr;
    bool gather = false;
};
// Runs the product over T tokens. Where `ws` (dense_workspace_floats() floats) is given and the output is OUT_RESIDUAL,
// a decode-sized product may come back as K-slices for the next norm to add instead; without a dst it always does (one
// slice or more, and ws holds at least T * n floats).
size_t dense_workspace_floats();
Slices dense(hipStream_t s, int arith, const DenseJob & job, int T, float * ws);

// ---- the tokens of a step by sequence ---------------------------------------------------------------
// The tokens of one sequence in a step, in order: run_tok[start .. start + n) are flat token indices.
struct SeqRun { int32_t slot, start, n, flags; };      // flags bit 0: the sequence starts here (state is zero), bit 1: the
                                                       // plane of the slot's convolution inputs that holds the current ones
struct SeqRuns {
    const SeqRun * runs = nullptr;
    int n = 0, longest = 0, shortest = 0;
    const int32_t * tok = nullptr;
};

// ---- norms ----------------------------------------------------------------------------------------
enum : int { NORM_RMS = 0, NORM_LAYER = 1 };
// act[i] = norm(x[rows[i]] (+ slices + the row of `plus`, written back)) * w; statistics and products in f32. With
// act_rows the same activations also as plain rows of act_kf * 32.
void norm_act(hipStream_t s, int arith, int kind, float * x, const float * w, int E, float eps, const int32_t * rows,
              int n_rows, void * act, int act_kf, const Slices & add, const float * plus = nullptr, void * act_rows = nullptr);
// x[t][:] += the slices, for a stream that is read elsewhere than in the next norm.
void add_slices(hipStream_t s, float * x, int E, int T, const Slices & add);
// x[copy][t] = scale * embed[tok[t]] for `copies` planes `stride` floats apart (bf16 rows of E).
void embed_rows(hipStream_t s, const uint16_t * embed, const int32_t * tok, int E, float scale, int T, float * x, int copies, size_t stride);

// Several residual streams x_1 .. x_n of [T][E] floats (hyper-connections). A sublayer reads u = sum_a in[a] x_a; what it
// leaves, y, changes every stream at once: x_b <- sum_a mix[a][b] x_a + out[b] y. A sublayer's weights: in[n], out[n], mix[n][n].
constexpr int MAX_STREAMS = 16;
constexpr int stream_weights(int n) { return n * (n + 2); }
struct Streams {
    float * x = nullptr;
    int n = 0;
    size_t stride = 0;             // floats from one stream to the next
};
// First the streams take in the slices of y by the weights `done` of the sublayer that left them (null: nothing is due), then
// act[i] = norm(u[rows[i]]) * w with u read by the weights `next` (null: u is the streams' plain sum). RMS norm; act_rows as in norm_act.
void streams_norm_act(hipStream_t s, int arith, const Streams & x, const float * done, const Slices & y, const float * next,
                      const float * w, int E, float eps, const int32_t * rows, int n_rows, void * act, int act_kf, void * act_rows = nullptr);
// out[t] = the sum of the streams once they have taken in y, which they do not here.
void streams_sum(hipStream_t s, const Streams & x, const float * done, const Slices & y, int E, int T, float * out);

// Norms before and after each sublayer, RMS norms in `groups` equal consecutive parts of the row, each by its own root mean
// square. First x[t] += mult * norm(slices) * after, written back (after null: no norm; no slices: x stays; rows: only
// x[rows[i]] is read, and nothing written back). Then, with w, h[t] = norm(x[t]) * w goes to act, and with act_rows also to
// plain rows. With taps it goes there as h_t + sum over j of taps[j] h_(t - n_taps + 1 + j), zeros before the sequence starts, a
// causal convolution over the tokens of each run whose inputs from earlier steps lie in `history` as in ShortConv.
struct SublayerNorm {
    float * x = nullptr;
    int E = 0, groups = 1;
    float eps = 0.0f, mult = 1.0f;
    Slices add;
    const float * after = nullptr, * w = nullptr;
    const int32_t * rows = nullptr;
    void * act = nullptr, * act_rows = nullptr;
    int act_kf = 0;
    const float * taps = nullptr;  // [n_taps][E], the last row the current token's
    int n_taps = 0;
    float * history = nullptr;     // [2 planes][slots][n_taps - 1][E]
    size_t plane = 0;
    SeqRuns runs;
    float * h = nullptr;           // scratch [T][E], for runs of more than one token
};
void sublayer_norm(hipStream_t s, int arith, const SublayerNorm & n, int n_rows);

// x[t] = norm(scale * embed[tok[t]] + pairs[row]) * w, groups as above; row is (previous token * mul_prev + token * mul_cur) mod
// buckets, and `buckets` for a sequence's first token. The last token of a run is left in `last` for the next step.
struct PairEmbedding {
    const uint16_t * embed = nullptr, * pairs = nullptr;      // bf16 rows of E
    const int32_t * tok = nullptr;
    float scale = 1.0f;
    int64_t buckets = 0, mul_prev = 0, mul_cur = 0;
    const float * w = nullptr;
    int E = 0, groups = 1;
    float eps = 0.0f;
    SeqRuns runs;
    float * last = nullptr;        // [2 planes][slots]
    size_t plane = 0;
    float * x = nullptr;
};
void embed_pairs(hipStream_t s, const PairEmbedding & e, int T);

// ---- attention ---------------------------------------------------------------------------------------
// A page of a cache: PAGE tokens x kf fragments of 32 columns, f16 or f32,
//   [column / 32][token / 16][lane = 16 * ((column % 32) / 8) + token % 16][column % 8]
// (several key/value heads: one head's fragments behind the other's). Fragments a head's row of `columns` columns is
// stored in: the widths the attention kernel is compiled for, zero padded.
int cache_frags(int columns);
// ... of a head's key row and its value row where their widths differ.
struct PairFrags { int k, v; };
PairFrags pair_frags(int key_columns, int value_columns);
constexpr size_t cache_page_elems(int kf) { return (size_t)kf * 32 * PAGE; }
// Queries' latent: act_q = RMS norm of proj[t][0, q_rank) times q_w. With kv_w also the cached latent: RMS norm of
// proj[t][kv_col, kv_col + kv_rank) times kv_w into cell[t] of the pool.
struct LatentNorms {
    const float * proj = nullptr;
    int ld = 0, q_rank = 0, kv_col = 0, kv_rank = 0;
    const float * q_w = nullptr, * kv_w = nullptr;
    float eps = 0.0f;
    void * act_q = nullptr;
    int act_q_kf = 0;
    void * pool = nullptr;
    int pool_kf = 0;
    const int32_t * cell = nullptr;
};
void latent_norms(hipStream_t s, int arith, const LatentNorms & a, int T);

// Grouped attention's rows between the input product and the cache, where they cannot leave in the product's epilogue:
// proj[t] holds H queries of dim columns from q_col on, G keys and G values (vdim columns) from k_col and v_col on. Queries and keys
// are RMS normed over all their heads at once (q_w, k_w), then the first `pairs` pairs (2 i, 2 i + 1) of each head rotated:
// queries to rows [t][H][kf * 32], keys to their cells. Values go to their cells mixed with those of the same token in
// `first`, (1 - share) v + share first; without `share`, first (where given) receives them.
struct HeadRows {
    const float * proj = nullptr;
    int ld = 0, H = 0, G = 0, dim = 0, vdim = 0, q_col = 0, k_col = 0, v_col = 0;
    const float * q_w = nullptr, * k_w = nullptr;
    float eps = 0.0f;
    int pairs = 0;
    const float * table = nullptr;             // [T][pairs][2]: cosine and sine
    const float * share = nullptr;             // one value
    float * first = nullptr;                   // [T][G * vdim]
    void * q = nullptr, * k_pool = nullptr, * v_pool = nullptr;
    int kf = 0, vf = 0;
    const int32_t * cell = nullptr;
};
void head_rows(hipStream_t s, int arith, const HeadRows & a, int T);

// Attention over paged caches: absorbed queries over latents (v_pool null, one head's worth of rows that are keys and
// values at once), or grouped attention over keys and values of G heads. A block serves up to `block_cols` of the
// T x (H / G) query columns (token-major) of one row of the step, for every key/value head.
struct AttnBlock { int32_t row, col0; };         // row of the step, first of its n * (H / G) columns
struct StackAttn {
    const void * q = nullptr;      // [T][H][kf * 32]; latents: already scaled by scale * log2(e)
    int H = 0, G = 1, kf = 0, vf = 0;            // fragments of a head's keys and of its values (latents: the same)
    int window = 0, chunk = 0;     // positions seen: the last `window`, or those of the same chunk of positions (0: no bound)
    float scale = 1.0f, softcap = 0.0f;          // with v_pool: score = scale * q.k, then softcap * tanh(score / softcap)
    const RowDesc * rows = nullptr;
    const AttnBlock * blocks = nullptr;
    int n_blocks = 0, block_cols = 0, splits = 1;
    const int32_t * table = nullptr;
    int max_pages = 0;
    const void * pool = nullptr, * v_pool = nullptr;
    void * partial = nullptr;      // several splits: [T * H][splits][vf * 32] means in f16 ...
    float * partial_ml = nullptr;  // ... and [T * H][splits][2] maxima and sums (stack_partial_floats() for both)
    void * out = nullptr;          // activations: column h * vf * 32 + c
    int out_kf = 0;
};
int stack_block_cols(int arith, int cols_per_token, int kf, int vf, bool pair, int n_tokens, int n_rows);
// Workgroups that share a block's keys, given the longest resident span among the step's rows.
int stack_splits(int arith, const StackAttn & a, int max_resident);
size_t stack_partial_floats(int T, int H, int vf, int splits);
void stack_attention(hipStream_t s, int arith, const StackAttn & a);
void stack_combine(hipStream_t s, const StackAttn & a, int T);      // of several splits (nothing to do for one)

// ---- rotary positions ----------------------------------------------------------------------------------
// table[t][i] = magnitude * (cos, sin)(pos[t] * freq[i]) for i < pairs; angles in double.
void rotary_table(hipStream_t s, const double * freq, int pairs, double magnitude, const int32_t * pos, int T, float * table);

// ---- expert routing --------------------------------------------------------------------------------------
// Per token the `top` experts of largest logit (ties to the lower index), with several groups of neighbouring experts among
// those of the `keep` groups whose largest logit is largest. Their weights: `scale` times the softmax over the chosen logits,
// the softmax over all of them, or each logit's sigmoid. Then the pairs sorted by expert into slots, every expert from a multiple of 16 on, cut into tiles of
// `block` slots.
constexpr int MAX_EXPERTS = 1024, MAX_TOP = 64;
enum : int { SCORE_OVER_CHOSEN = 0, SCORE_OVER_ALL, SCORE_SIGMOID };
struct ExpertRoute {
    const float * logits = nullptr;            // [T][ld]
    int ld = 0, experts = 0, top = 0, block = 0;
    int groups = 1, keep = 1;
    int score = SCORE_OVER_CHOSEN;
    float scale = 1.0f;
    int32_t * sel = nullptr;                   // [T * top]
    float * weight = nullptr;                  // [T * top]
    int32_t * slot_pair = nullptr;             // [expert_slots()]
    int32_t * tiles = nullptr, * n_tiles = nullptr;
};
int expert_block(int arith, int T, int top, int experts);
size_t expert_slots(int T, int top, int experts);            // with room for a whole last tile
int expert_max_tiles(int T, int top, int experts, int block);
void expert_route(hipStream_t s, const ExpertRoute & r, int T);

// Page copies and cell gathers of any pool of pages (elem bytes 2 or 4).
void stack_copy_page(hipStream_t s, void * pool, size_t page_bytes, int src, int dst);
void stack_cells(hipStream_t s, void * pool, int kf, int elem, const int32_t * cells, int n, void * rows, bool gather);

// ---- recurrent mixers ---------------------------------------------------------------------------------
// Short causal convolution over time per channel, then SiLU: out[t][c] from the taps newest last, zeros before a sequence
// starts. Runs of fewer than `least` tokens are left out.
struct ShortConv {
    SeqRuns runs;
    int channels = 0, taps = 0, least = 0;
    const float * in = nullptr;    // [T][ld], the channels side by side
    int ld = 0;
    const float * w = nullptr, * b = nullptr;            // [channels][taps]; bias per channel or none
    float * state = nullptr;       // [2 planes][slots][taps - 1][channels]
    size_t plane = 0;              // floats of a plane
    float * out = nullptr;         // [T][channels]
};
void short_conv(hipStream_t s, const ShortConv & c);

// ---- state-space mixer (Mamba-2) ------------------------------------------------------------------------
struct MambaShape {
    int heads = 0, vdim = 0, state = 0, groups = 0, taps = 0, norm_groups = 0;
    constexpr int inner() const { return heads * vdim; }
    constexpr int channels() const { return inner() + 2 * groups * state; }
    constexpr int rows() const { return inner() + channels() + heads; }      // of the input projection
};
struct MambaJob {
    MambaShape sh;
    const float * proj = nullptr;  // [T][ld]: z | x | B | C | dt
    int ld = 0;
    const float * conv_w = nullptr, * conv_b = nullptr, * dt_bias = nullptr, * A_log = nullptr, * D = nullptr, * norm_w = nullptr;
    float eps = 0.0f;
    SeqRuns runs;
    float * conv_state = nullptr;  // [2 planes][slots][taps - 1][channels]
    size_t conv_plane = 0;         // floats of a plane
    float * state = nullptr;       // [slots][heads][state][vdim]
    float * xbc = nullptr;         // scratch [T][channels]
    float * y = nullptr;           // scratch [T][inner]
    void * out = nullptr;          // activations, inner wide
    int out_kf = 0;
};
void mamba_mix(hipStream_t s, int arith, const MambaJob & j, int T);

// ---- matrix states with a rule of writing: gated delta rules, linear attention with a forget gate -------------
// Per head a state S [dim][vdim], decayed, written to and read out: S <- g * S (rows scaled), S <- S + k u^T, o = S^T q.
// Delta rules: u = beta (v - S^T k); q and k unit vectors per key/value head (q also times dim^-1/2) and, like v, convolved and
// through SiLU before; beta a sigmoid per head; g = exp(-exp(A_log) softplus(a + dt_bias)), a value per head and row of the state
// (RULE_DELTA_CHANNELS) or one per head (RULE_DELTA_HEADS).
// RULE_FORGET: what a row forgets is what it writes, g = lower + (1 - lower) sigmoid(z), k = 1 - g, u = v, q through SiLU; no
// convolution.
// The read-out of a head: o / rms(o) * norm_w, times the sigmoid or SiLU of a gate where there is one.
enum : int { RULE_DELTA_CHANNELS = 0, RULE_DELTA_HEADS, RULE_FORGET };
enum : int { GATE_NONE = 0, GATE_SIGMOID, GATE_SILU };
struct DeltaShape {
    int rule = RULE_DELTA_CHANNELS, gate = GATE_SIGMOID;
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 1;
    int decay_rank = 0, gate_rank = 0;         // inner widths of the projections of a and gate, where they have one
    constexpr int keys() const { return kv_heads * dim; }
    constexpr int inner() const { return heads * vdim; }
    constexpr int channels() const { return 2 * keys() + inner(); }       // q | k (forget rule: z) | v
    constexpr int vpitch() const { return (vdim + 3) / 4 * 4; }            // of a row of the state
    constexpr size_t state_floats() const { return (size_t)heads * dim * vpitch(); }
};
struct DeltaJob {
    DeltaShape sh;
    const float * proj = nullptr;  // [T][ld]: q | k | v | beta (heads)
    int ld = 0;
    const float * decay = nullptr, * gate = nullptr;     // [T][ld_low]: a (heads x dim, or heads), gate (heads x vdim)
    int ld_low = 0;
    const float * conv_w = nullptr, * A_log = nullptr, * dt_bias = nullptr, * lower = nullptr, * norm_w = nullptr;
    float eps = 0.0f, unit_eps = 0.0f;
    SeqRuns runs;
    float * conv_state = nullptr;  // as in ShortConv
    size_t conv_plane = 0;
    float * state = nullptr;       // [slots][heads][dim][vpitch]
    float * qkv = nullptr;         // scratch [T][channels]
    float * y = nullptr;           // scratch [T][inner]
    float * chunks = nullptr;      // scratch, delta_chunk_floats()
    void * out = nullptr;          // activations, inner wide
    int out_kf = 0;
};
size_t delta_chunk_floats(const DeltaShape & sh, int T, int n_runs);
void delta_mix(hipStream_t s, int arith, const DeltaJob & j, int T);

void copy_floats(hipStream_t s, const float * src, float * dst, size_t n);

}  // namespace rk
