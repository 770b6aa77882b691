// Layer-stack models in the engine: loading a checkpoint folder, the cache pools and recurrent state of every pass
// through a layer, the step's plan for them and the forward pass. Slots, pages, packing, sampling, sequence operations and the
// generators are the engine's own (engine.cpp, generate.cpp).
#include "engine.hpp"
#include "safetensors_file.hpp"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <tuple>

namespace retro {

namespace {

void hip_check(hipError_t err, const char * what) {
    if (err != hipSuccess) throw std::runtime_error(std::string("HIP error in ") + what + ": " + hipGetErrorString(err));
}

constexpr float kGateSlope = 1.702f;           // of the clamped gated pair's sigmoid
constexpr float kUnitEps = 1e-6f;              // under the root of the delta rule's unit vectors

int up16(int n) { return (n + 15) / 16 * 16; }
int up32(int n) { return (n + 31) / 32 * 32; }

// Uploads a checkpoint's tensors and lays matrices out for the dense kernels.
class Loader {
public:
    Loader(const SafetensorsFile & f, hipStream_t s) : file_(f), stream_(s) {}

    std::vector<float> floats(const std::string & name, const std::vector<int64_t> & shape) {
        const StTensor & t = file_.require(name, shape);
        const size_t n = t.nbytes / (t.dtype == "F32" ? 4 : 2);
        std::vector<float> v(n);
        if (t.dtype == "F32") {
            std::memcpy(v.data(), t.data, n * 4);
        } else if (t.dtype == "BF16") {
            for (size_t i = 0; i < n; ++i) {
                uint16_t b;
                std::memcpy(&b, t.data + 2 * i, 2);
                const uint32_t w = (uint32_t)b << 16;
                std::memcpy(&v[i], &w, 4);
            }
        } else {
            throw std::runtime_error("tensor " + name + " must be BF16 or F32");
        }
        return v;
    }
    static void upload(const std::vector<float> & v, DevBuf & out) {
        out.alloc(v.size() * 4);
        if (!v.empty()) hip_check(hipMemcpy(out.ptr, v.data(), v.size() * 4, hipMemcpyHostToDevice), "hipMemcpy");
    }
    void vector(const std::string & name, const std::vector<int64_t> & shape, DevBuf & out, float plus = 0.0f) {
        std::vector<float> v = floats(name, shape);
        for (float & x : v) x += plus;
        upload(v, out);
    }
    // Several tensors one behind the other.
    void vectors(const std::vector<std::pair<std::string, std::vector<int64_t>>> & parts, DevBuf & out) {
        std::vector<float> all;
        for (const auto & p : parts) {
            const std::vector<float> v = floats(p.first, p.second);
            all.insert(all.end(), v.begin(), v.end());
        }
        upload(all, out);
    }
    // Raw rows that are gathered.
    void table(const std::string & name, int rows, int cols, DevBuf & out) {
        const StTensor & t = file_.require(name, {rows, cols});
        if (t.dtype != "BF16") throw std::runtime_error("tensor " + name + " must be BF16");
        out.alloc(t.nbytes);
        hip_check(hipMemcpy(out.ptr, t.data, t.nbytes, hipMemcpyHostToDevice), "hipMemcpy");
    }
    // Taps [channels][taps] of a convolution, tap by tap.
    void taps(const std::string & name, int channels, int taps, DevBuf & out) {
        const std::vector<float> v = floats(name, {channels, taps});
        std::vector<float> w(v.size());
        for (int c = 0; c < channels; ++c)
            for (int j = 0; j < taps; ++j) w[(size_t)j * channels + c] = v[(size_t)c * taps + j];
        upload(w, out);
    }
    // Biases of a matrix's rows, each tensor at its rows' places.
    void biases(const StackLayer::Matrix & m, const std::vector<std::tuple<std::string, int, rk::PackMap>> & parts, DevBuf & out) {
        std::vector<float> all((size_t)m.w.batch * m.w.tiles * 16, 0.0f);
        for (const auto & p : parts) {
            const rk::PackMap & at = std::get<2>(p);
            const std::vector<float> v = floats(std::get<0>(p), {std::get<1>(p)});
            for (int r = 0; r < (int)v.size(); ++r) all[(size_t)(at.at + r / at.run * at.step + r % at.run)] = v[(size_t)r];
        }
        upload(all, out);
    }
    // Rows of a matrix of `cols` columns.
    int rows_of(const std::string & name, int cols) {
        const StTensor * t = file_.find(name);
        if (!t) throw std::runtime_error("model is missing tensor " + name);
        if (t->shape.size() != 2 || t->shape[0] < 1 || t->shape[0] > (1 << 24) || t->shape[1] != cols) throw std::runtime_error("tensor " + name + " has an unexpected shape");
        return (int)t->shape[0];
    }
    void shape(StackLayer::Matrix & m, int n, int kf, int batch = 1) {
        m.w.n = n;
        m.w.tiles = (n + 15) / 16;
        m.w.kf = kf;
        m.w.batch = batch;
        m.buf.alloc(m.w.bytes());
        hip_check(hipMemsetAsync(m.buf.ptr, 0, m.w.bytes(), stream_), "hipMemsetAsync");
        m.w.w = m.buf.as<uint16_t>();
    }
    // The tensor [rows][cols] on the device as stored; valid until the next call.
    const uint16_t * raw(const std::string & name, int rows, int cols) {
        const StTensor & t = file_.require(name, {rows, cols});
        if (t.dtype != "BF16") throw std::runtime_error("tensor " + name + " must be BF16");
        hip_check(hipStreamSynchronize(stream_), "hipStreamSynchronize");
        raw_.ensure(t.nbytes);
        hip_check(hipMemcpyAsync(raw_.ptr, t.data, t.nbytes, hipMemcpyHostToDevice, stream_), "hipMemcpyAsync");
        return raw_.as<uint16_t>();
    }
    // ... as rows of batch b of m.
    void matrix(const std::string & name, int rows, int cols, StackLayer::Matrix & m, rk::PackMap row = 0, rk::PackMap col = 0, int b = 0) {
        rk::dense_pack(stream_, raw(name, rows, cols), rows, cols, cols, 1, m.buf.as<uint16_t>() + b * rk::frag_weight_elems(m.w.tiles, m.w.kf), m.w.kf, row, col);
    }
    // A gate and an up matrix as row tiles in turn, from row tile tile0 on.
    void gated(const std::string & p, int rows, int cols, StackLayer::Matrix & m, int tile0 = 0, int b = 0) {
        matrix(p + "gate", rows, cols, m, gate_row(tile0), 0, b);
        matrix(p + "up", rows, cols, m, up_row(tile0), 0, b);
    }
    static rk::PackMap gate_row(int tile0 = 0) { return {tile0 * 16, 16, 32}; }
    static rk::PackMap up_row(int tile0 = 0) { return {tile0 * 16 + 16, 16, 32}; }
    static int gated_rows(int ff) { return 2 * up16(ff); }
    // The rows of `heads` heads from row0 on, every head padded, the columns of a rotated pair (i and i + rotated / 2) side by side.
    void heads(const std::string & name, int heads, int dim, int padded, int rotated, int cols, StackLayer::Matrix & m, int row0) {
        const uint16_t * src = raw(name, heads * dim, cols);
        for (int h = 0; h < heads; ++h)
            each_part(dim, rotated, [&](int from, int n, int to, int step) {
                rk::dense_pack(stream_, src + ((size_t)h * dim + from) * cols, n, cols, cols, 1, m.buf.as<uint16_t>(), m.w.kf, {row0 + h * padded + to, 1, step}, 0);
            });
    }
    // ... and their biases.
    void head_biases(const std::string & name, int heads, int dim, int padded, int rotated, int row0, std::vector<float> & all) {
        const std::vector<float> v = floats(name, {heads * dim});
        for (int h = 0; h < heads; ++h)
            each_part(dim, rotated, [&](int from, int n, int to, int step) {
                for (int i = 0; i < n; ++i) all[(size_t)(row0 + h * padded + to + i * step)] = v[(size_t)(h * dim + from + i)];
            });
    }
    // ... and the columns of a matrix that reads them.
    void from_heads(const std::string & name, int rows, int heads, int dim, int padded, int rotated, StackLayer::Matrix & m) {
        const uint16_t * src = raw(name, rows, heads * dim);
        for (int h = 0; h < heads; ++h)
            each_part(dim, rotated, [&](int from, int n, int to, int step) {
                rk::dense_pack(stream_, src + h * dim + from, rows, n, heads * dim, 1, m.buf.as<uint16_t>(), m.w.kf, 0, {h * padded + to, 1, step});
            });
    }
    void finish() { hip_check(hipStreamSynchronize(stream_), "hipStreamSynchronize"); }

private:
    template <typename F> static void each_part(int dim, int rotated, F f) {
        if (rotated > 0) {
            f(0, rotated / 2, 0, 2);
            f(rotated / 2, rotated / 2, 1, 2);
        }
        if (dim > rotated) f(rotated, dim - rotated, rotated, 1);
    }
    const SafetensorsFile & file_;
    hipStream_t stream_;
    DevBuf raw_;
};

}  // namespace

void Engine::load_stack(const std::string & path) {
    if (ggml_activations_) throw std::runtime_error("RETRO_ACTIVATIONS=ggml is an arithmetic of GGUF models");
    if (cfg_.kv_dtype == RETRO_ENGINE_KV_DTYPE_F16) arith_ = rk::ARITH_16;
    else if (cfg_.kv_dtype == RETRO_ENGINE_KV_DTYPE_F32) arith_ = rk::ARITH_32;
    else throw std::runtime_error("layer-stack models run with kv_dtype F16 (bf16 products) or F32 (everything in f32)");
    stack_.reset(new StackConfig(StackConfig::read(path)));
    const StackConfig & c = *stack_;
    SafetensorsFile file(path + "/model.safetensors");
    Loader ld(file, stream_);
    hp_.arch = c.arch->name;
    hp_.n_layer = (int)c.runs.size();
    hp_.n_embd = c.width;
    hp_.n_vocab = c.vocab;
    hp_.eps = c.eps;
    const int E = c.width, KE = rk::frags_of(E);

    ld.table("embed", c.vocab, E, tok_embd_.buf);
    tok_embd_.w.type = rk::WT_BF16;
    tok_embd_.w.K = E;
    tok_embd_.w.N = c.vocab;
    tok_embd_.w.bytes = tok_embd_.buf.bytes;
    tok_embd_.w.raw = tok_embd_.buf.as<uint8_t>();
    if (c.arch->norm_after) ld.table("bigram", (int)c.pair_buckets + 1, E, pair_embd_);
    ld.shape(stack_head_, c.vocab, KE);
    ld.matrix(c.arch->own_head ? "head" : "embed", c.vocab, E, stack_head_);
    const float norm_plus = c.arch->norm_around_one ? 1.0f : 0.0f;
    ld.vector("final.norm", {E}, out_norm_, norm_plus);
    if (c.arch->norm_after) ld.vector("embed.norm", {E}, embed_norm_);

    stack_layers_.resize(c.layers.size());
    for (size_t l = 0; l < c.layers.size(); ++l) {
        StackLayer & L = stack_layers_[l];
        L.spec = c.layers[l];
        const LayerSpec & sp = L.spec;
        const std::string p = "l" + std::to_string(l) + ".", m = p + "mix.";
        const bool parallel = c.arch->parallel;
        if (parallel && sp.moe.experts > 0) throw std::runtime_error("experts in parallel layers are not supported");
        if (parallel && sp.mixer == Mixer::DELTA) throw std::runtime_error("matrix states in parallel layers are not supported");
        for (int q = 0; q < (sp.has_ff() ? 2 : 1) && c.streams > 0; ++q) {
            const std::string hc = p + (q == 0 ? "hc1." : "hc2.");
            ld.vectors({{hc + "in", {c.streams}}, {hc + "out", {c.streams}}, {hc + "mix", {c.streams, c.streams}}}, L.hyper[q]);
        }
        ld.vector(p + "norm1", {E}, L.norm, norm_plus);
        if (!parallel && sp.has_ff()) ld.vector(p + "norm2", {E}, L.norm2, norm_plus);
        for (int q = 0; q < (sp.has_ff() ? 2 : 1); ++q) {
            const std::string n = std::to_string(q + 1);
            if (c.arch->norm_after) ld.vector(p + "norm" + n + "b", {E}, L.after[q], norm_plus);
            if (c.input_taps > 0) ld.taps(p + "canon" + n, E, c.input_taps, L.taps[q]);
        }
        if (c.arch->layer_scale) {
            ld.vector(p + "ls1", {E}, L.scale_mix);
            if (sp.ff > 0) ld.vector(p + "ls2", {E}, L.scale_ff);
        }
        // input rows: the mixer's, in whole tiles, then a parallel feed-forward's
        const LatentSpec & a = sp.latent;
        const AttentionSpec & ga = sp.attention;
        const rk::PairFrags head = ga.frags();
        rk::DeltaShape & ds = L.spec.delta;
        const bool own_values = !c.arch->keys_are_values, in_place = c.arch->rows_in_place();
        const int rotated = c.arch->pairs == Pairs::HALVES ? ga.rot.dims : 0;      // columns of a head whose pairs are brought together
        int beside = parallel ? sp.ff : 0;              // rows behind the mixer's that go elsewhere
        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            const bool own = a.kv_from < 0;
            L.kv_col = up16(a.q_rank);
            L.gate_col = L.kv_col + (own ? up16(a.kv_rank) : 0);
            L.in_rows = L.gate_col + a.heads;
        } else if (sp.grouped_attention() && in_place) {
            L.k_col = ga.heads * head.k * 32;
            L.v_col = L.k_col + ga.kv_heads * head.k * 32;
            L.in_rows = L.v_col + (own_values ? ga.kv_heads * head.v * 32 : 0);
            if (sp.mixer == Mixer::ATTENTION_MAMBA2) beside = sp.mamba.rows();
        } else if (sp.grouped_attention()) {
            L.k_col = up16(ga.heads * ga.dim);
            L.v_col = L.k_col + up16(ga.kv_heads * ga.dim);
            L.in_rows = L.v_col + ga.kv_heads * ga.vdim;
        } else if (sp.mixer == Mixer::DELTA && ds.rule == rk::RULE_FORGET) {
            L.in_rows = ds.channels();
        } else if (sp.mixer == Mixer::DELTA && ds.rule == rk::RULE_DELTA_HEADS) {
            L.decay_col = ds.channels() + ds.heads;
            L.gate_col = L.decay_col + ds.heads;
            L.in_rows = L.gate_col + ds.inner();
        } else if (sp.mixer == Mixer::DELTA) {
            ds.decay_rank = ld.rows_of(m + "a1", E);
            ds.gate_rank = ld.rows_of(m + "g1", E);
            L.low_frags = std::max(rk::frags_of(ds.decay_rank), rk::frags_of(ds.gate_rank));
            L.in_rows = ds.channels() + ds.heads;
            beside = L.low_frags * 32 + ds.gate_rank;
        } else {
            L.in_rows = sp.mamba.rows();
        }
        L.in_tiles = (L.in_rows + 15) / 16;
        ld.shape(L.w_in, beside > 0 ? L.in_tiles * 16 + beside : L.in_rows, KE);
        if (parallel && beside > 0) ld.matrix(p + "mlp.up", beside, E, L.w_in, L.in_tiles * 16);
        const int mix = sp.mix_width(), KM = rk::frags_of(mix);
        const bool two = sp.mixer == Mixer::ATTENTION_MAMBA2;
        const std::string am = m + (two ? "left." : ""), sm = m + (two ? "right." : "");      // attention's tensors, Mamba-2's
        ld.shape(L.w_out, E, KM + rk::frags_of(parallel ? beside : sp.beside_width()));
        if (sp.grouped_attention()) ld.from_heads(am + "o", E, ga.heads, ga.vdim, head.v * 32, own_values ? 0 : rotated, L.w_out);
        else ld.matrix(m + "o", E, mix, L.w_out);
        if (two) {
            ld.matrix(sm + "o", E, sp.beside_width(), L.w_out, 0, KM * 32);
            Loader::upload(std::vector<float>((size_t)E, sp.left_scale), L.scale_mix);
            Loader::upload(std::vector<float>((size_t)E, sp.right_scale), L.scale_ff);
        }
        if (sp.grouped_attention() && c.arch->out_bias) {
            std::vector<float> b((size_t)L.w_out.w.tiles * 16, 0.0f);
            ld.head_biases(am + "o.b", 1, E, 0, 0, 0, b);
            for (float & x : b) x *= sp.left_scale;
            Loader::upload(b, L.out_bias);
        }
        if (parallel && beside > 0) ld.matrix(p + "mlp.down", E, beside, L.w_out, 0, KM * 32);
        if (!parallel && sp.ff > 0) {
            if (rk::out_is_glu(c.arch->ff_act)) {
                ld.shape(L.ff_in, Loader::gated_rows(sp.ff), KE);
                ld.gated(p + "mlp.", sp.ff, E, L.ff_in);
            } else {
                ld.shape(L.ff_in, sp.ff, KE);
                ld.matrix(p + "mlp.up", sp.ff, E, L.ff_in);
            }
            ld.shape(L.ff_out, E, rk::frags_of(sp.ff));
            ld.matrix(p + "mlp.down", E, sp.ff, L.ff_out);
            if (c.arch->ff_bias) {
                if (rk::out_is_glu(c.arch->ff_act)) ld.biases(L.ff_in, {{p + "mlp.gate.b", sp.ff, Loader::gate_row()}, {p + "mlp.up.b", sp.ff, Loader::up_row()}}, L.ff_in_bias);
                else ld.biases(L.ff_in, {{p + "mlp.up.b", sp.ff, 0}}, L.ff_in_bias);
                ld.biases(L.ff_out, {{p + "mlp.down.b", E, 0}}, L.ff_out_bias);
            }
        } else if (sp.moe.experts > 0) {
            const MoeSpec & e = sp.moe;
            const std::string sh = p + "mlp.shared.";
            const int route = e.experts + (e.shared_ff > 0 && c.arch->shared_gate ? 1 : 0);
            L.route_tiles = up32(route) / 16;
            ld.shape(L.ff_in, e.shared_ff > 0 ? L.route_tiles * 16 + Loader::gated_rows(e.shared_ff) : route, KE);
            ld.matrix(p + "mlp.router", e.experts, E, L.ff_in);
            if (e.shared_ff > 0) {
                if (c.arch->shared_gate) ld.matrix(sh + "sg", 1, E, L.ff_in, e.experts);
                ld.gated(sh, e.shared_ff, E, L.ff_in, L.route_tiles);
                ld.shape(L.ff_out, E, rk::frags_of(e.shared_ff));
                ld.matrix(sh + "down", E, e.shared_ff, L.ff_out);
            }
            ld.shape(L.experts_in, Loader::gated_rows(e.ff), KE, e.experts);
            ld.shape(L.experts_out, E, rk::frags_of(e.ff), e.experts);
            for (int x = 0; x < e.experts; ++x) {
                const std::string ex = p + "mlp.e" + std::to_string(x) + ".";
                ld.gated(ex, e.ff, E, L.experts_in, 0, x);
                ld.matrix(ex + "down", E, e.ff, L.experts_out, 0, 0, x);
            }
        }

        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            ld.matrix(m + "dq", a.q_rank, E, L.w_in);
            ld.vector(m + "dq.norm", {a.q_rank}, L.q_norm);
            if (a.kv_from < 0) {
                ld.matrix(m + "dkv", a.kv_rank, E, L.w_in, L.kv_col);
                ld.vector(m + "dkv.norm", {a.kv_rank}, L.kv_norm);
            }
            ld.matrix(m + "g", a.heads, E, L.w_in, L.gate_col);
            // queries head by head, every head padded to whole fragments
            const int D = up32(a.dim), R = 32 * rk::cache_frags(a.kv_rank);
            ld.shape(L.uq, a.heads * D, rk::frags_of(a.q_rank));
            const uint16_t * uq = ld.raw(m + "uq", a.heads * a.dim, a.q_rank);
            for (int h = 0; h < a.heads; ++h)
                rk::dense_pack(stream_, uq + (size_t)h * a.dim * a.q_rank, a.dim, a.q_rank, a.q_rank, 1, L.uq.buf.as<uint16_t>(), L.uq.w.kf, h * D, 0);
            // absorption: row r of head h holds column r of the head's key up-projection
            ld.shape(L.uk, R, D / 32, a.heads);
            const uint16_t * uk = ld.raw(m + "uk", a.heads * a.dim, a.kv_rank);
            const size_t uk_head = rk::frag_weight_elems(L.uk.w.tiles, L.uk.w.kf);
            for (int h = 0; h < a.heads; ++h)
                rk::dense_pack(stream_, uk + (size_t)h * a.dim * a.kv_rank, a.kv_rank, a.dim, 1, a.kv_rank, L.uk.buf.as<uint16_t>() + h * uk_head, L.uk.w.kf, 0, 0);
            ld.shape(L.uv, a.vdim, R / 32, a.heads);
            const uint16_t * uv = ld.raw(m + "uv", a.heads * a.vdim, a.kv_rank);
            const size_t uv_head = rk::frag_weight_elems(L.uv.w.tiles, L.uv.w.kf);
            for (int h = 0; h < a.heads; ++h)
                rk::dense_pack(stream_, uv + (size_t)h * a.vdim * a.kv_rank, a.vdim, a.kv_rank, a.kv_rank, 1, L.uv.buf.as<uint16_t>() + h * uv_head, L.uv.w.kf, 0, 0);
        } else if (sp.grouped_attention()) {
            if (!in_place) {
                const int nq = ga.heads * ga.dim, nk = ga.kv_heads * ga.dim, nv = ga.kv_heads * ga.vdim;
                ld.matrix(m + "q", nq, E, L.w_in);
                ld.matrix(m + "k", nk, E, L.w_in, L.k_col);
                ld.matrix(m + "v", nv, E, L.w_in, L.v_col);
                ld.biases(L.w_in, {{m + "q.b", nq, 0}, {m + "k.b", nk, L.k_col}, {m + "v.b", nv, L.v_col}}, L.in_bias);
                ld.vector(m + "q.norm", {nq}, L.q_norm);
                ld.vector(m + "k.norm", {nk}, L.kv_norm);
                if (ga.v_mix && !ga.v_first) ld.vector(m + "vmix", {}, L.v_share);
            } else {
                ld.heads(am + "q", ga.heads, ga.dim, head.k * 32, rotated, E, L.w_in, 0);
                ld.heads(am + "k", ga.kv_heads, ga.dim, head.k * 32, rotated, E, L.w_in, L.k_col);
                if (own_values) {
                    ld.heads(am + "v", ga.kv_heads, ga.vdim, head.v * 32, 0, E, L.w_in, L.v_col);
                    std::vector<float> b((size_t)L.w_in.w.tiles * 16, 0.0f);
                    ld.head_biases(am + "q.b", ga.heads, ga.dim, head.k * 32, rotated, 0, b);
                    ld.head_biases(am + "k.b", ga.kv_heads, ga.dim, head.k * 32, rotated, L.k_col, b);
                    ld.head_biases(am + "v.b", ga.kv_heads, ga.vdim, head.v * 32, 0, L.v_col, b);
                    Loader::upload(b, L.in_bias);
                }
            }
            for (size_t r = 0; r < rotary_.size(); ++r) if (rotary_[r].spec == ga.rot) L.rotary = (int)r;
            if (L.rotary < 0) {
                L.rotary = (int)rotary_.size();
                rotary_.emplace_back();
                RotaryTable & t = rotary_.back();
                t.spec = ga.rot;
                const std::vector<double> f = ga.rot.frequencies();
                t.freq.alloc(f.size() * sizeof(double));
                if (!f.empty()) hip_check(hipMemcpy(t.freq.ptr, f.data(), t.freq.bytes, hipMemcpyHostToDevice), "hipMemcpy");
            }
        } else if (sp.mixer == Mixer::DELTA && ds.rule == rk::RULE_FORGET) {
            ld.matrix(m + "q", ds.keys(), E, L.w_in);
            ld.matrix(m + "f", ds.keys(), E, L.w_in, ds.keys());
            ld.matrix(m + "v", ds.inner(), E, L.w_in, 2 * ds.keys());
            ld.biases(L.w_in, {{m + "f.b", ds.keys(), ds.keys()}}, L.in_bias);
            const std::vector<float> lower = ld.floats(m + "lower", {ds.keys()});
            for (float x : lower) if (!(x >= 0.0f && x <= 1.0f)) throw std::runtime_error("tensor " + m + "lower must lie between 0 and 1");
            Loader::upload(lower, L.lower);
            ld.vector(m + "norm", {ds.vdim}, L.gate_norm);
        } else if (sp.mixer == Mixer::DELTA && ds.rule == rk::RULE_DELTA_HEADS) {
            ld.matrix(m + "q", ds.keys(), E, L.w_in);
            ld.matrix(m + "k", ds.keys(), E, L.w_in, ds.keys());
            ld.matrix(m + "v", ds.inner(), E, L.w_in, 2 * ds.keys());
            ld.matrix(m + "b", ds.heads, E, L.w_in, ds.channels());
            ld.matrix(m + "a", ds.heads, E, L.w_in, L.decay_col);
            ld.matrix(m + "g", ds.inner(), E, L.w_in, L.gate_col);
            ld.vectors({{m + "q.conv", {ds.keys(), ds.taps}}, {m + "k.conv", {ds.keys(), ds.taps}}, {m + "v.conv", {ds.inner(), ds.taps}}}, L.conv_w);
            ld.vector(m + "dt_bias", {ds.heads}, L.dt_bias);
            ld.vector(m + "A_log", {ds.heads}, L.A_log);
            ld.vector(m + "norm", {ds.vdim}, L.gate_norm);
        } else if (sp.mixer == Mixer::DELTA) {
            const int at_a = L.in_tiles * 16, decays = ds.heads * ds.dim, gates = ds.inner();
            ld.matrix(m + "q", ds.keys(), E, L.w_in);
            ld.matrix(m + "k", ds.keys(), E, L.w_in, ds.keys());
            ld.matrix(m + "v", ds.inner(), E, L.w_in, 2 * ds.keys());
            ld.matrix(m + "b", ds.heads, E, L.w_in, ds.channels());
            ld.matrix(m + "a1", ds.decay_rank, E, L.w_in, at_a);
            ld.matrix(m + "g1", ds.gate_rank, E, L.w_in, at_a + L.low_frags * 32);
            ld.shape(L.low, std::max(decays, gates), L.low_frags, 2);
            ld.matrix(m + "a2", decays, ds.decay_rank, L.low, 0, 0, 0);
            ld.matrix(m + "g2", gates, ds.gate_rank, L.low, 0, 0, 1);
            ld.vectors({{m + "q.conv", {ds.keys(), ds.taps}}, {m + "k.conv", {ds.keys(), ds.taps}}, {m + "v.conv", {ds.inner(), ds.taps}}}, L.conv_w);
            ld.vector(m + "dt_bias", {decays}, L.dt_bias);
            ld.vector(m + "A_log", {ds.heads}, L.A_log);
            ld.vector(m + "norm", {ds.vdim}, L.gate_norm);
        }
        if (sp.state_space()) {
            const rk::MambaShape & s = sp.mamba;
            ld.matrix(sm + "in", s.rows(), E, L.w_in, two ? L.in_tiles * 16 : 0);
            ld.vector(sm + "conv", {s.channels(), s.taps}, L.conv_w);
            ld.vector(sm + "conv.b", {s.channels()}, L.conv_b);
            ld.vector(sm + "dt_bias", {s.heads}, L.dt_bias);
            ld.vector(sm + "A_log", {s.heads}, L.A_log);
            ld.vector(sm + "D", {s.heads}, L.D);
            ld.vector(sm + "norm", {s.inner()}, L.gate_norm);
        }
    }
    ld.finish();
    vocab_.tokenizer_error = "a checkpoint folder holds no vocabulary";

    uint64_t hash = UINT64_C(14695981039346656037);
    auto mix_in = [&hash](const void * data, size_t n) {
        const unsigned char * b = (const unsigned char *)data;
        for (size_t i = 0; i < n; ++i) { hash ^= b[i]; hash *= UINT64_C(1099511628211); }
    };
    mix_in(path.data(), path.size());
    const uint64_t size = file.tensor_bytes();
    mix_in(&size, sizeof(size));
    fingerprint_ = hash;
}

// Cache pools, recurrent state and the step's buffers.
void Engine::build_stack() {
    const StackConfig & c = *stack_;
    const size_t n_run = c.runs.size(), elem = (size_t)arith_;
    const int B = (int)cfg_.n_batch, E = c.width, n_slots = (int)cfg_.n_seq_max;
    qt_ = 0;                                  // attention plans its own blocks
    stack_runs_.resize(n_run);
    k_pool_.resize(n_run);
    v_pool_.resize(n_run);
    // per run: a pool of latents, or one of keys and one of values
    struct Pool { size_t at = 0, bytes = 0; };
    std::vector<Pool> pools(2 * n_run);
    std::vector<int> last(c.layers.size(), 0);              // the latest run of a layer
    size_t total = 0;
    auto pool = [&](size_t run, bool v, int kf) {
        Pool & p = pools[2 * run + v];
        p.bytes = (size_t)n_pages_ * rk::cache_page_elems(kf) * elem;
        p.at = total;
        total += (p.bytes + 255) / 256 * 256;
        cache_parts_.push_back({(int)run, v, (size_t)kf * 32 * elem});
    };
    for (size_t r = 0; r < n_run; ++r) {
        StackRun & R = stack_runs_[r];
        R.layer = c.runs[r].layer;
        R.add_embedding = c.runs[r].add_embedding;
        looped_ |= R.add_embedding;
        last[(size_t)R.layer] = (int)r;
        R.pool = (int)r;
        const LayerSpec & sp = c.layers[(size_t)R.layer];
        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            if (sp.latent.kv_from >= 0) R.pool = last[(size_t)sp.latent.kv_from];
            else pool(r, false, rk::cache_frags(sp.latent.kv_rank));
        } else if (sp.grouped_attention()) {
            const rk::PairFrags f = sp.attention.frags();
            for (int v = 0; v < 2; ++v) pool(r, v != 0, sp.attention.kv_heads * (v ? f.v : f.k));
        }
    }
    kv_slab_.alloc(total);
    if (total) hip_check(hipMemsetAsync(kv_slab_.ptr, 0, total, stream_), "hipMemsetAsync");      // pages never hold non-finite values
    for (size_t i = 0; i < pools.size(); ++i)
        if (pools[i].bytes) (i & 1 ? v_pool_ : k_pool_)[i / 2] = PoolView{(uint8_t *)kv_slab_.ptr + pools[i].at, pools[i].bytes};

    // recurrent state: states [part][slot], then two planes of what convolutions and embeddings remember [part][slot], each
    // part from a multiple of four floats on
    auto part = [&](float * & base, size_t slot, bool planes) {
        if (slot > 0) state_parts_.push_back({&base, slot, planes});
    };
    for (StackRun & R : stack_runs_) {
        const LayerSpec & sp = c.layers[(size_t)R.layer];
        const rk::MambaShape & s = sp.mamba;
        const rk::DeltaShape & d = sp.delta;
        if (sp.mixer == Mixer::DELTA) {
            part(R.state, d.state_floats(), false);
            part(R.conv_state, (size_t)(d.taps - 1) * d.channels(), true);
        } else if (sp.state_space()) {
            part(R.state, (size_t)s.heads * s.state * s.vdim, false);
            part(R.conv_state, (size_t)(s.taps - 1) * s.channels(), true);
        }
        for (int q = 0; q < (sp.has_ff() ? 2 : 1) && c.input_taps > 0; ++q) part(R.history[q], (size_t)(c.input_taps - 1) * E, true);
    }
    if (c.arch->norm_after) part(last_token_, 1, true);
    auto held = [&](const StatePart & p) { return (p.slot * n_slots + 3) / 4 * 4; };
    size_t states = 0;
    for (const StatePart & p : state_parts_) {
        (p.planes ? conv_plane_floats_ : states) += held(p);
        recurrent_slot_floats_ += p.slot;
    }
    recurrent_slab_.alloc((states + 2 * conv_plane_floats_) * 4);
    if (recurrent_slab_.ptr) {
        hip_check(hipMemsetAsync(recurrent_slab_.ptr, 0, recurrent_slab_.bytes, stream_), "hipMemsetAsync");
        float * st = recurrent_slab_.as<float>(), * cv = st + states;
        for (const StatePart & p : state_parts_) {
            float * & at = p.planes ? cv : st;
            *p.base = at;
            at += held(p);
        }
    }

    build_pack_buffers();
    build_step_buffers();
    const double magnitude = 1.0;             // no rotation: only the factor the packing kernel reads
    inv_freq_.alloc(sizeof(double));
    hip_check(hipMemcpy(inv_freq_.ptr, &magnitude, sizeof(double), hipMemcpyHostToDevice), "hipMemcpy");

    size_t h = rk::frag_elems(B, rk::frags_of(E)), cq = 0, q = 0, qa = 0, ol = 0, mix = 0, ff = 0, xbc = 0, y = 0;
    auto zeroed = [&](DevBuf & b, size_t n) {       // padding that no producer writes has to be finite
        b.alloc(n);
        if (n) hip_check(hipMemsetAsync(b.ptr, 0, n, stream_), "hipMemsetAsync");
    };
    size_t route = 0, pairs = 0, slots = 0, tiles = 0, expert_h = 0, first = 0, low = 0, decay = 0, chunks = 0, beside = 0;
    for (const StackLayer & L : stack_layers_) {
        const LayerSpec & sp = L.spec;
        mix = std::max(mix, rk::frag_elems(B, rk::frags_of(sp.mix_width())));
        if (sp.ff > 0) ff = std::max(ff, rk::frag_elems(B, rk::frags_of(sp.ff)));
        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            const LatentSpec & a = sp.latent;
            cq = std::max(cq, rk::frag_elems(B, rk::frags_of(a.q_rank)));
            q = std::max(q, rk::frag_elems(B, a.heads * rk::frags_of(a.dim)));
            qa = std::max(qa, (size_t)B * a.heads * 32 * rk::cache_frags(a.kv_rank));
            ol = std::max(ol, rk::frag_elems(B, a.heads * rk::cache_frags(a.kv_rank)));
        } else if (sp.grouped_attention()) {
            const AttentionSpec & a = sp.attention;
            qa = std::max(qa, (size_t)B * a.heads * 32 * a.frags().k);
            if (a.v_mix) first = std::max(first, (size_t)B * a.kv_heads * a.vdim);
        } else if (sp.mixer == Mixer::DELTA) {
            const rk::DeltaShape & d = sp.delta;
            xbc = std::max(xbc, (size_t)B * d.channels());
            y = std::max(y, (size_t)B * d.inner());
            if (d.rule == rk::RULE_DELTA_CHANNELS) {
                low = std::max(low, rk::frag_elems(B, 2 * L.low_frags));
                decay = std::max(decay, (size_t)B * 2 * up16(L.low.w.n));
            }
            chunks = std::max(chunks, rk::delta_chunk_floats(d, B, n_slots));
        }
        if (sp.state_space()) {
            xbc = std::max(xbc, (size_t)B * sp.mamba.channels());
            y = std::max(y, (size_t)B * sp.mamba.inner());
            if (sp.beside_width() > 0) beside = std::max(beside, rk::frag_elems(B, rk::frags_of(sp.beside_width())));
        }
        if (sp.moe.experts > 0) {
            const MoeSpec & e = sp.moe;
            const size_t n = rk::expert_slots(B, e.top, e.experts);
            if (e.shared_ff > 0) ff = std::max(ff, rk::frag_elems(B, rk::frags_of(e.shared_ff)));
            route = std::max(route, (size_t)B * up32(e.experts + 1));
            pairs = std::max(pairs, (size_t)B * e.top);
            slots = std::max(slots, n);
            tiles = std::max(tiles, (size_t)rk::expert_max_tiles(B, e.top, e.experts, 16));
            expert_h = std::max(expert_h, rk::frag_elems((int)n, rk::frags_of(e.ff)));
            moe_ws_floats_ = std::max(moe_ws_floats_, (size_t)B * E * e.top);
        }
    }
    for (const StackLayer & L : stack_layers_)        // what of the input product does not go to its place at once
        st_proj_ld_ = std::max(st_proj_ld_, !L.spec.grouped_attention() || !c.arch->rows_in_place() ? L.in_tiles * 16 : (L.w_in.w.tiles - L.in_tiles) * 16);
    for (RotaryTable & t : rotary_) t.table.alloc((size_t)B * t.spec.dims * 4);
    if (looped_) st_embed_.alloc((size_t)B * E * 4);
    if (route) zeroed(st_rows_, (size_t)B * rk::frags_of(E) * 32 * elem);
    st_route_.alloc(route * 4);
    ex_sel_.alloc(pairs * 4);
    ex_weight_.alloc(pairs * 4);
    ex_slot_.alloc(slots * 4);
    if (tiles) ex_tiles_.alloc((tiles + 1) * 16);           // the count behind the tiles
    x_.alloc((size_t)B * E * 4 * std::max(c.streams, 1));
    st_first_.alloc(first * 4);
    zeroed(st_beside_, beside * elem);
    if (c.input_taps > 0) st_in_rows_.alloc((size_t)B * E * 4);
    zeroed(st_low_, low * elem);
    zeroed(st_decay_, decay * 4);
    st_chunks_.alloc(chunks * 4);
    zeroed(st_h_, h * elem);
    zeroed(st_out_, h * elem);
    zeroed(st_proj_, (size_t)B * st_proj_ld_ * 4);
    zeroed(st_cq_, cq * elem);
    zeroed(st_q_, q * elem);
    zeroed(st_qa_, qa * elem);
    zeroed(st_ol_, ol * elem);
    zeroed(st_mix_, mix * elem);
    zeroed(st_ff_, ff * elem);
    zeroed(st_xbc_, xbc * 4);
    zeroed(st_y_, y * 4);
    zeroed(ex_h_, expert_h * elem);
    mm_ws_.alloc((std::max(rk::dense_workspace_floats(), c.streams > 0 || c.around() ? (size_t)B * E : 0) + moe_ws_floats_) * 4);
}

// ---- recurrent state of a slot --------------------------------------------------------------------

void Engine::state_copy(int32_t src, int32_t dst) {
    const int plane = slots_[(size_t)src].plane;
    slots_[(size_t)dst].plane = 0;
    for (const StatePart & p : state_parts_)
        rk::copy_floats(stream_, *p.base + (p.planes ? plane * conv_plane_floats_ : 0) + src * p.slot, *p.base + dst * p.slot, p.slot);
}

void Engine::state_pack(int32_t slot, float * out) {
    const int plane = slots_[(size_t)slot].plane;
    for (const StatePart & p : state_parts_) {
        hip_check(hipMemcpyAsync(out, *p.base + (p.planes ? plane * conv_plane_floats_ : 0) + slot * p.slot, p.slot * 4, hipMemcpyDeviceToHost, stream_), "hipMemcpyAsync");
        out += p.slot;
    }
    hip_check(hipStreamSynchronize(stream_), "seq_save");
}

void Engine::state_unpack(int32_t slot, const float * in) {
    slots_[(size_t)slot].plane = 0;
    for (const StatePart & p : state_parts_) {
        hip_check(hipMemcpyAsync(*p.base + slot * p.slot, in, p.slot * 4, hipMemcpyHostToDevice, stream_), "hipMemcpyAsync");
        in += p.slot;
    }
    hip_check(hipStreamSynchronize(stream_), "seq_load");
}

// ---- the step's plan ------------------------------------------------------------------------------
// Blocks of query columns for every number of columns per token (heads of a key/value head) among the layers, and for recurrent models the tokens of every sequence
// in order (a step may hold several rows of one slot).

void Engine::plan_stack(const std::vector<RowView> & rows, const std::vector<std::pair<int, int>> & before) {
    block_plans_.clear();
    plan_blocks_.clear();
    plan_runs_.clear();
    plan_run_tok_.clear();
    plan_max_run_ = plan_min_run_ = 0;
    step_rows_ = (int)rows.size();
    int total = 0;
    for (const RowView & r : rows) total += (int)r.n;
    for (const LayerSpec & sp : stack_->layers) {
        if (!sp.attends()) continue;
        const bool pair = sp.grouped_attention();
        const int H = pair ? sp.attention.heads / sp.attention.kv_heads : sp.latent.heads, R = rk::cache_frags(std::max(sp.latent.kv_rank, 1));
        const rk::PairFrags f = pair ? sp.attention.frags() : rk::PairFrags{R, R};
        const int cols = rk::stack_block_cols(arith_, H, f.k, f.v, pair, total, (int)rows.size());
        if (std::any_of(block_plans_.begin(), block_plans_.end(), [&](const BlockPlan & b) { return b.heads == H && b.cols == cols; })) continue;
        BlockPlan plan{H, cols, plan_blocks_.size(), 0};
        for (size_t r = 0; r < rows.size(); ++r)
            for (int64_t c = 0; c < (int64_t)rows[r].n * H; c += plan.cols) plan_blocks_.push_back({(int32_t)r, (int32_t)c});
        plan.n = plan_blocks_.size() - plan.first;
        block_plans_.push_back(plan);
    }
    if (!is_hybrid()) return;
    std::vector<int> run_of(slots_.size(), -1);
    std::vector<std::vector<int32_t>> toks;
    int32_t at = 0;
    for (const RowView & r : rows) {
        int & k = run_of[(size_t)r.slot];
        if (k < 0) {
            k = (int)plan_runs_.size();
            Slot & s = slots_[(size_t)r.slot];
            const bool fresh = before[(size_t)r.slot].second <= before[(size_t)r.slot].first;
            plan_runs_.push_back({r.slot, 0, 0, (fresh ? 1 : 0) | (s.plane << 1)});
            s.plane = 1 - s.plane;            // this step leaves what the next one remembers in the other plane
            toks.emplace_back();
        }
        for (uint32_t i = 0; i < r.n; ++i) toks[(size_t)k].push_back(at + (int32_t)i);
        at += (int32_t)r.n;
    }
    for (size_t k = 0; k < plan_runs_.size(); ++k) {
        plan_runs_[k].start = (int32_t)plan_run_tok_.size();
        plan_runs_[k].n = (int32_t)toks[k].size();
        plan_max_run_ = std::max(plan_max_run_, plan_runs_[k].n);
        plan_min_run_ = k == 0 ? plan_runs_[k].n : std::min(plan_min_run_, plan_runs_[k].n);
        plan_run_tok_.insert(plan_run_tok_.end(), toks[k].begin(), toks[k].end());
    }
}

size_t Engine::stack_plan_bytes() const {
    return plan_runs_.size() * sizeof(rk::SeqRun) + plan_blocks_.size() * sizeof(rk::AttnBlock) + plan_run_tok_.size() * 4;
}

void Engine::stage_stack_plan(uint8_t * host, const uint8_t * device) {
    size_t at = 0;
    auto put = [&](const void * src, size_t n) {
        if (n) std::memcpy(host + at, src, n);
        const uint8_t * d = device + at;
        at += n;
        return d;
    };
    d_runs_ = (const rk::SeqRun *)put(plan_runs_.data(), plan_runs_.size() * sizeof(rk::SeqRun));
    d_blocks_ = (const rk::AttnBlock *)put(plan_blocks_.data(), plan_blocks_.size() * sizeof(rk::AttnBlock));
    d_run_tok_ = (const int32_t *)put(plan_run_tok_.data(), plan_run_tok_.size() * 4);
}

// ---- the forward pass -------------------------------------------------------------------------------

// Attention over the caches of `at`, its blocks and splits filled in here.
void Engine::attend(rk::StackAttn & at, int T) {
    size_t pt = prof_begin(PC_ATTN);
    const int per_token = at.H / at.G, cols = rk::stack_block_cols(arith_, per_token, at.kf, at.vf, at.v_pool != nullptr, T, step_rows_);
    const BlockPlan * plan = nullptr;
    for (const BlockPlan & b : block_plans_) if (b.heads == per_token && b.cols == cols) plan = &b;
    at.rows = d_stage_.as<rk::RowDesc>();
    at.blocks = d_blocks_ + plan->first;
    at.n_blocks = (int)plan->n;
    at.block_cols = plan->cols;
    at.table = table_.as<int32_t>();
    at.max_pages = max_pages_;
    at.splits = rk::stack_splits(arith_, at, step_max_resident_);
    st_partial_.ensure(rk::stack_partial_floats(T, at.H, at.vf, at.splits) * 4);
    at.partial_ml = st_partial_.as<float>();
    at.partial = at.partial_ml + (size_t)T * at.H * at.splits * 2;
    rk::stack_attention(stream_, arith_, at);
    prof_end(PC_ATTN, pt);
    if (at.splits > 1) {
        pt = prof_begin(PC_COMBINE);
        rk::stack_combine(stream_, at, T);
        prof_end(PC_COMBINE, pt);
    }
}

void Engine::mix_latent(const StackLayer & L, const StackRun & run, int T) {
    const LatentSpec & a = L.spec.latent;
    const int D = rk::frags_of(a.dim), R = rk::cache_frags(a.kv_rank), H = a.heads, ld = st_proj_ld_;
    float * proj = st_proj_.as<float>(), * ws = mm_ws_.as<float>();
    void * pool = k_pool_[(size_t)run.pool].ptr;
    size_t pt = prof_begin(PC_ROPE);
    rk::LatentNorms n;
    n.proj = proj; n.ld = ld; n.q_rank = a.q_rank; n.kv_col = L.kv_col; n.kv_rank = a.kv_rank;
    n.q_w = L.q_norm.as<float>(); n.kv_w = L.kv_norm.as<float>(); n.eps = stack_->eps;
    n.act_q = st_cq_.ptr; n.act_q_kf = rk::frags_of(a.q_rank);
    n.pool = pool; n.pool_kf = R; n.cell = pk_.cell;
    rk::latent_norms(stream_, arith_, n, T);
    prof_end(PC_ROPE, pt);
    pt = prof_begin(PC_ABSORB);
    rk::DenseJob uq;
    uq.w = L.uq.w;
    uq.x = {st_cq_.ptr, rk::frags_of(a.q_rank), 0};
    uq.a.kind = rk::OUT_ACT; uq.a.dst = st_q_.ptr; uq.a.ld = H * D;
    rk::dense(stream_, arith_, uq, T, ws);
    rk::DenseJob uk;
    uk.w = L.uk.w;
    uk.x = {st_q_.ptr, H * D, D};
    uk.a.kind = rk::OUT_QUERY; uk.a.dst = st_qa_.ptr; uk.a.ld = R * 32; uk.a.col_batch = H;
    uk.a.scale = (float)((double)a.scale * 1.4426950408889634);      // the softmax runs on powers of two
    rk::dense(stream_, arith_, uk, T, ws);
    prof_end(PC_ABSORB, pt);
    rk::StackAttn at;
    at.q = st_qa_.ptr; at.H = H; at.kf = at.vf = R; at.window = a.window;
    at.pool = pool;
    at.out = st_ol_.ptr; at.out_kf = H * R;
    attend(at, T);
    pt = prof_begin(PC_OPROJ);
    rk::DenseJob uv;
    uv.w = L.uv.w;
    uv.x = {st_ol_.ptr, H * R, R};
    uv.a.kind = rk::OUT_ACT_GATED; uv.a.dst = st_mix_.ptr; uv.a.ld = rk::frags_of(L.spec.mix_width()); uv.a.col_batch = a.vdim;
    uv.a.gate = proj + L.gate_col; uv.a.ld_gate = ld;
    rk::dense(stream_, arith_, uv, T, ws);
    prof_end(PC_OPROJ, pt);
}

void Engine::mix_mamba(const StackLayer & L, const StackRun & run, int T, void * out) {
    const size_t pt = prof_begin(PC_SCAN);
    rk::MambaJob j;
    j.sh = L.spec.mamba;
    j.proj = st_proj_.as<float>(); j.ld = st_proj_ld_;
    j.conv_w = L.conv_w.as<float>(); j.conv_b = L.conv_b.as<float>(); j.dt_bias = L.dt_bias.as<float>();
    j.A_log = L.A_log.as<float>(); j.D = L.D.as<float>(); j.norm_w = L.gate_norm.as<float>();
    j.eps = stack_->eps;
    j.runs = step_runs();
    j.conv_state = run.conv_state; j.conv_plane = conv_plane_floats_; j.state = run.state;
    j.xbc = st_xbc_.as<float>(); j.y = st_y_.as<float>();
    j.out = out; j.out_kf = rk::frags_of(L.spec.mamba.inner());
    rk::mamba_mix(stream_, arith_, j, T);
    prof_end(PC_SCAN, pt);
}

rk::SeqRuns Engine::step_runs() const {
    rk::SeqRuns r;
    r.runs = d_runs_; r.n = (int)plan_runs_.size(); r.longest = plan_max_run_; r.shortest = plan_min_run_; r.tok = d_run_tok_;
    return r;
}

// The input product has left queries, keys, values and write strengths as f32 rows, decays and gates behind them, or the inner
// columns of decays and gates as activations.
void Engine::mix_delta(const StackLayer & L, const StackRun & run, int T) {
    const rk::DeltaShape & sh = L.spec.delta;
    rk::DeltaJob j;
    j.sh = sh;
    j.proj = st_proj_.as<float>(); j.ld = st_proj_ld_;
    if (sh.rule == rk::RULE_DELTA_CHANNELS) {
        const size_t pt = prof_begin(PC_LOW_RANK);
        const int half = up16(L.low.w.n);
        rk::DenseJob low;
        low.w = L.low.w;
        low.x = {st_low_.ptr, 2 * L.low_frags, L.low_frags};
        low.a.kind = rk::OUT_F32; low.a.dst = st_decay_.ptr; low.a.ld = 2 * half; low.a.col_batch = half;
        rk::dense(stream_, arith_, low, T, nullptr);
        j.decay = st_decay_.as<float>(); j.gate = j.decay + half; j.ld_low = 2 * half;
        prof_end(PC_LOW_RANK, pt);
    } else if (sh.rule == rk::RULE_DELTA_HEADS) {
        j.decay = j.proj + L.decay_col; j.gate = j.proj + L.gate_col; j.ld_low = st_proj_ld_;
    }
    const size_t pt = prof_begin(PC_SCAN);
    j.conv_w = L.conv_w.as<float>(); j.A_log = L.A_log.as<float>(); j.dt_bias = L.dt_bias.as<float>(); j.lower = L.lower.as<float>();
    j.norm_w = L.gate_norm.as<float>();
    j.eps = stack_->eps; j.unit_eps = kUnitEps;
    j.runs = step_runs();
    j.conv_state = run.conv_state; j.conv_plane = conv_plane_floats_; j.state = run.state;
    j.qkv = st_xbc_.as<float>(); j.y = st_y_.as<float>(); j.chunks = st_chunks_.as<float>();
    j.out = st_mix_.ptr; j.out_kf = rk::frags_of(L.spec.mix_width());
    rk::delta_mix(stream_, arith_, j, T);
    prof_end(PC_SCAN, pt);
}

// Grouped attention. The input product has already left queries, keys and values in their places, unless queries and keys are
// still to be normed: then all come as f32 rows.
void Engine::mix_attention(const StackLayer & L, const StackRun & run, int T) {
    const AttentionSpec & a = L.spec.attention;
    const rk::PairFrags f = a.frags();
    void * keys = k_pool_[(size_t)run.pool].ptr, * values = v_pool_[(size_t)run.pool].ptr;
    if (!stack_->arch->rows_in_place()) {
        const size_t pt = prof_begin(PC_ROPE);
        const RotaryTable & t = rotary_[(size_t)L.rotary];
        rk::HeadRows r;
        r.proj = st_proj_.as<float>(); r.ld = st_proj_ld_;
        r.H = a.heads; r.G = a.kv_heads; r.dim = a.dim; r.vdim = a.vdim; r.k_col = L.k_col; r.v_col = L.v_col;
        r.q_w = L.q_norm.as<float>(); r.k_w = L.kv_norm.as<float>(); r.eps = stack_->eps;
        r.pairs = t.spec.dims / 2; r.table = t.table.as<float>();
        if (a.v_mix) r.first = st_first_.as<float>();
        if (a.v_mix && !a.v_first) r.share = L.v_share.as<float>();
        r.q = st_qa_.ptr; r.k_pool = keys; r.v_pool = values;
        r.kf = f.k; r.vf = f.v; r.cell = pk_.cell;
        rk::head_rows(stream_, arith_, r, T);
        prof_end(PC_ROPE, pt);
    }
    rk::StackAttn at;
    at.q = st_qa_.ptr; at.H = a.heads; at.G = a.kv_heads; at.kf = f.k; at.vf = f.v;
    at.window = a.window; at.chunk = a.chunk;
    at.scale = a.scale; at.softcap = a.softcap;
    at.pool = keys; at.v_pool = values;
    at.out = st_mix_.ptr; at.out_kf = a.heads * f.v;
    attend(at, T);
}

// The feed-forward of a sequential layer over the normed rows in st_h_.
rk::Slices Engine::stack_feed_forward(const StackLayer & L, int T) {
    const StackConfig & c = *stack_;
    const int E = c.width, KE = rk::frags_of(E), KF = rk::frags_of(L.spec.ff);
    float * ws = mm_ws_.as<float>();
    if (L.spec.moe.experts > 0) return stack_experts(L, T);
    size_t pt = prof_begin(PC_GATEUP);
    rk::DenseJob in;
    in.w = L.ff_in.w;
    in.x = {st_h_.ptr, KE, 0};
    in.a.kind = c.arch->ff_act; in.a.dst = st_ff_.ptr; in.a.ld = KF;
    in.a.limit = L.spec.ff_limit; in.a.slope = kGateSlope;
    in.bias = L.ff_in_bias.as<float>();
    rk::dense(stream_, arith_, in, T, ws);
    prof_end(PC_GATEUP, pt);
    pt = prof_begin(PC_DOWN);
    rk::DenseJob out;
    out.w = L.ff_out.w;
    out.x = {st_ff_.ptr, KF, 0};
    out.kf1 = KF;
    out.a.kind = rk::OUT_RESIDUAL; out.a.dst = c.streams > 0 || c.around() ? nullptr : x_.ptr; out.a.ld = E;
    out.bias = L.ff_out_bias.as<float>();
    const rk::Slices left = rk::dense(stream_, arith_, out, T, ws);
    prof_end(PC_DOWN, pt);
    return left;
}

// Router and shared expert in one product, the routing, the chosen experts; every choice leaves a slice of the residual.
rk::Slices Engine::stack_experts(const StackLayer & L, int T) {
    const StackConfig & c = *stack_;
    const MoeSpec & e = L.spec.moe;
    const int E = c.width, KE = rk::frags_of(E), KS = rk::frags_of(std::max(e.shared_ff, 1)), KX = rk::frags_of(e.ff);
    float * ws = mm_ws_.as<float>(), * route = st_route_.as<float>();
    const int ld = up32(e.experts + 1);
    size_t pt = prof_begin(PC_SHARED);
    rk::DenseJob in;
    in.w = L.ff_in.w;
    in.x = {st_h_.ptr, KE, 0};
    in.split_tile = L.route_tiles;
    in.n_a = e.experts + (e.shared_ff > 0 && c.arch->shared_gate ? 1 : 0);
    in.a.kind = rk::OUT_F32; in.a.dst = route; in.a.ld = ld;
    in.b.kind = c.arch->expert_act; in.b.dst = st_ff_.ptr; in.b.ld = KS;
    in.b.limit = e.shared_limit; in.b.slope = kGateSlope;
    rk::dense(stream_, arith_, in, T, ws);
    prof_end(PC_SHARED, pt);
    pt = prof_begin(PC_ROUTE);
    rk::ExpertRoute r;
    r.logits = route; r.ld = ld; r.experts = e.experts; r.top = e.top;
    r.block = rk::expert_block(arith_, T, e.top, e.experts);
    r.groups = e.groups; r.keep = e.keep; r.score = c.arch->score; r.scale = e.scale;
    r.sel = ex_sel_.as<int32_t>(); r.weight = ex_weight_.as<float>(); r.slot_pair = ex_slot_.as<int32_t>();
    r.tiles = ex_tiles_.as<int32_t>();
    r.n_tiles = r.tiles + (ex_tiles_.bytes / 16 - 1) * 4;
    rk::expert_route(stream_, r, T);
    prof_end(PC_ROUTE, pt);
    rk::ExpertGroups g;
    g.tiles = r.tiles; g.n_tiles = r.n_tiles; g.block = r.block; g.max_tiles = rk::expert_max_tiles(T, e.top, e.experts, r.block);
    g.slot_pair = r.slot_pair; g.weight = r.weight; g.top = e.top; g.pairs = T * e.top;
    g.weigh_input = c.arch->weigh_input;
    pt = prof_begin(PC_EXPERTS_IN);
    rk::DenseJob up;
    up.w = L.experts_in.w;
    up.x = {st_rows_.ptr, KE, 0};
    up.groups = &g;
    up.gather = true;
    up.a.kind = c.arch->expert_act; up.a.dst = ex_h_.ptr; up.a.ld = KX;
    up.a.limit = e.limit; up.a.slope = kGateSlope;
    rk::dense(stream_, arith_, up, T, ws);
    prof_end(PC_EXPERTS_IN, pt);
    rk::Slices left;
    if (e.shared_ff > 0) {
        pt = prof_begin(PC_SHARED);
        rk::DenseJob out;
        out.w = L.ff_out.w;
        out.x = {st_ff_.ptr, KS, 0};
        out.kf1 = KS;
        out.a.kind = rk::OUT_RESIDUAL; out.a.dst = c.streams > 0 || c.around() ? nullptr : x_.ptr; out.a.ld = E;
        if (c.arch->shared_gate) { out.token_gate = route + e.experts; out.ld_token_gate = ld; }
        left = rk::dense(stream_, arith_, out, T, ws);
        prof_end(PC_SHARED, pt);
    }
    pt = prof_begin(PC_EXPERTS_OUT);
    const size_t slice = (size_t)T * E;
    rk::DenseJob down;
    down.w = L.experts_out.w;
    down.x = {ex_h_.ptr, KX, 0};
    down.groups = &g;
    down.a.kind = rk::OUT_EXPERT; down.a.dst = ws + (size_t)left.n * slice; down.a.ld = E; down.a.stride = slice;
    rk::dense(stream_, arith_, down, T, ws);
    prof_end(PC_EXPERTS_OUT, pt);
    left.data = ws;
    left.n += e.top;
    left.stride = slice;
    left.N = E;
    return left;
}

// The norm of a sublayer's output into the stream x.
rk::SublayerNorm Engine::around(float * x, const DevBuf * after, const rk::Slices & add) const {
    rk::SublayerNorm n;
    n.x = x; n.E = stack_->width; n.groups = stack_->norm_groups; n.eps = stack_->eps;
    n.mult = stack_->residual_mult;
    n.add = add;
    n.after = after ? after->as<float>() : nullptr;
    return n;
}

void Engine::forward_stack(int T, int n_out) {
    const StackConfig & c = *stack_;
    const int E = c.width, KE = rk::frags_of(E);
    float * x = x_.as<float>(), * ws = mm_ws_.as<float>();
    rk::Slices pending;                         // what the stream, or the streams by the weights `due`, have yet to take in
    const float * due = nullptr;
    const DevBuf * due_norm = nullptr;          // the norm that `pending` goes through
    rk::Streams streams;
    streams.x = x; streams.n = c.streams; streams.stride = (size_t)cfg_.n_batch * E;
    // the norm before a sublayer: the mixer (0) or the feed-forward (1) of a run
    auto norm = [&](const StackLayer & L, const StackRun & run, int q, const float * plus, void * act_rows) {
        const size_t pt = prof_begin(PC_NORM);
        const float * w = (q ? L.norm2 : L.norm).as<float>();
        if (c.around()) {
            rk::SublayerNorm n = around(x, due_norm, pending);
            n.w = w;
            n.act = st_h_.ptr; n.act_kf = KE; n.act_rows = act_rows;
            if (c.input_taps > 0) {
                n.taps = L.taps[q].as<float>(); n.n_taps = c.input_taps;
                n.history = run.history[q]; n.plane = conv_plane_floats_;
                n.runs = step_runs();
                n.h = st_in_rows_.as<float>();
            }
            rk::sublayer_norm(stream_, arith_, n, T);
        } else if (c.streams > 0) {
            rk::streams_norm_act(stream_, arith_, streams, due, pending, L.hyper[q].as<float>(), w, E, c.eps, nullptr, T, st_h_.ptr, KE, act_rows);
        } else {
            rk::norm_act(stream_, arith_, c.arch->norm, x, w, E, c.eps, nullptr, T, st_h_.ptr, KE, pending, plus, act_rows);
        }
        prof_end(PC_NORM, pt);
    };
    // what the sublayer q of L has left
    auto leave = [&](const StackLayer & L, int q, const rk::Slices & y) {
        pending = y;
        due = L.hyper[q].as<float>();
        due_norm = c.arch->norm_after ? &L.after[q] : nullptr;
    };
    size_t pt = prof_begin(PC_EMBED);
    if (c.arch->norm_after) {
        rk::PairEmbedding e;
        e.embed = (const uint16_t *)tok_embd_.w.raw; e.pairs = pair_embd_.as<uint16_t>();
        e.tok = pk_.tok; e.scale = c.embedding_scale;
        e.buckets = c.pair_buckets; e.mul_prev = c.pair_mul_prev; e.mul_cur = c.pair_mul_cur;
        e.w = embed_norm_.as<float>();
        e.E = E; e.groups = c.norm_groups; e.eps = c.eps;
        e.runs = step_runs();
        e.last = last_token_; e.plane = conv_plane_floats_;
        e.x = x;
        rk::embed_pairs(stream_, e, T);
    } else {
        rk::embed_rows(stream_, (const uint16_t *)tok_embd_.w.raw, pk_.tok, E, c.embedding_scale, T, x, std::max(c.streams, 1), streams.stride);
    }
    if (looped_) rk::copy_floats(stream_, x, st_embed_.as<float>(), (size_t)T * E);
    for (RotaryTable & t : rotary_)
        rk::rotary_table(stream_, t.freq.as<double>(), t.spec.dims / 2, t.spec.magnitude(), pk_.pos, T, t.table.as<float>());
    prof_end(PC_EMBED, pt);
    if (keep_residual_) {
        kept_residual_.ensure(stack_runs_.size() * (size_t)cfg_.n_batch * E * 4);
        kept_tokens_ = T;
    }
    for (size_t r = 0; r < stack_runs_.size(); ++r) {
        const StackRun & run = stack_runs_[r];
        const StackLayer & L = stack_layers_[(size_t)run.layer];
        const LayerSpec & sp = L.spec;
        const bool beside = c.arch->parallel && sp.ff > 0;
        norm(L, run, 0, run.add_embedding ? st_embed_.as<float>() : nullptr, nullptr);
        pt = prof_begin(PC_QKV);
        rk::DenseJob in;
        in.w = L.w_in.w;
        in.x = {st_h_.ptr, KE, 0};
        in.split_tile = L.in_tiles;
        in.n_a = L.in_rows;
        in.bias = L.in_bias.as<float>();
        if (sp.grouped_attention() && c.arch->rows_in_place()) {
            const AttentionSpec & a = sp.attention;
            const RotaryTable & t = rotary_[(size_t)L.rotary];
            in.a.kind = rk::OUT_ROTARY; in.a.dst = st_qa_.ptr;
            in.a.rot.H = a.heads; in.a.rot.G = a.kv_heads; in.a.rot.kf = a.frags().k; in.a.rot.vf = c.arch->keys_are_values ? 0 : a.frags().v; in.a.rot.pairs = t.spec.dims / 2;
            in.a.rot.table = t.table.as<float>();
            in.a.rot.k_pool = k_pool_[(size_t)run.pool].ptr; in.a.rot.v_pool = v_pool_[(size_t)run.pool].ptr;
            in.a.rot.cell = pk_.cell;
        } else {
            in.a.kind = rk::OUT_F32; in.a.dst = st_proj_.ptr; in.a.ld = st_proj_ld_;
        }
        if (sp.mixer == Mixer::ATTENTION_MAMBA2) {
            in.b.kind = rk::OUT_F32; in.b.dst = st_proj_.ptr; in.b.ld = st_proj_ld_;
        } else if (sp.mixer == Mixer::DELTA) {
            in.b.kind = rk::OUT_ACT; in.b.dst = st_low_.ptr; in.b.ld = 2 * L.low_frags;
        } else {
            in.b.kind = c.arch->ff_act; in.b.dst = st_ff_.ptr; in.b.ld = rk::frags_of(std::max(sp.ff, 1));
        }
        rk::dense(stream_, arith_, in, T, ws);
        prof_end(PC_QKV, pt);
        if (sp.mixer == Mixer::LATENT_ATTENTION) mix_latent(L, run, T);
        else if (sp.mixer == Mixer::DELTA) mix_delta(L, run, T);
        else if (sp.grouped_attention()) mix_attention(L, run, T);
        if (sp.state_space()) mix_mamba(L, run, T, sp.mixer == Mixer::MAMBA2 ? st_mix_.ptr : st_beside_.ptr);
        const int out_cat = c.arch->parallel ? PC_DOWN : PC_OPROJ, KM = rk::frags_of(sp.mix_width());
        pt = prof_begin(out_cat);
        rk::DenseJob out;
        out.w = L.w_out.w;
        out.x = {st_mix_.ptr, KM, 0};
        out.kf1 = KM;
        out.scale1 = L.scale_mix.as<float>();
        if (beside) {
            out.x2 = {st_ff_.ptr, rk::frags_of(sp.ff), 0};
            out.scale2 = L.scale_ff.as<float>();
        } else if (sp.mixer == Mixer::ATTENTION_MAMBA2) {
            out.x2 = {st_beside_.ptr, rk::frags_of(sp.beside_width()), 0};
            out.scale2 = L.scale_ff.as<float>();
        }
        out.bias = L.out_bias.as<float>();
        out.a.kind = rk::OUT_RESIDUAL; out.a.dst = c.streams > 0 || c.around() ? nullptr : x; out.a.ld = E;
        leave(L, 0, rk::dense(stream_, arith_, out, T, ws));
        prof_end(out_cat, pt);
        if (!c.arch->parallel && sp.has_ff()) {
            norm(L, run, 1, nullptr, sp.moe.experts > 0 ? st_rows_.ptr : nullptr);
            leave(L, 1, stack_feed_forward(L, T));
        }
        if (keep_residual_) {
            float * kept = kept_residual_.as<float>() + r * (size_t)cfg_.n_batch * E;
            if (c.streams > 0) {
                rk::streams_sum(stream_, streams, due, pending, E, T, kept);
            } else {
                rk::copy_floats(stream_, x, kept, (size_t)T * E);
                if (c.around()) rk::sublayer_norm(stream_, arith_, around(kept, due_norm, pending), T);
                else rk::add_slices(stream_, kept, E, T, pending);
            }
        }
    }
    if (n_out > 0) {
        logits_.ensure((size_t)n_out * c.vocab * 4);
        pt = prof_begin(PC_HEAD);
        if (c.around()) {
            rk::SublayerNorm n = around(x, due_norm, pending);
            n.w = out_norm_.as<float>();
            n.rows = pk_.out_tok;
            n.act = st_out_.ptr; n.act_kf = KE;
            rk::sublayer_norm(stream_, arith_, n, n_out);
        } else if (c.streams > 0) {
            rk::streams_norm_act(stream_, arith_, streams, due, pending, nullptr, out_norm_.as<float>(), E, c.eps, pk_.out_tok, n_out, st_out_.ptr, KE);
        } else {
            rk::norm_act(stream_, arith_, c.arch->norm, x, out_norm_.as<float>(), E, c.eps, pk_.out_tok, n_out, st_out_.ptr, KE, pending);
        }
        prof_end(PC_HEAD, pt);
        pt = prof_begin(PC_HEAD);
        rk::DenseJob head;
        head.w = stack_head_.w;
        head.x = {st_out_.ptr, KE, 0};
        head.a.kind = c.logit_softcap > 0.0f ? rk::OUT_F32_CAPPED : rk::OUT_F32; head.a.dst = logits_.ptr; head.a.ld = c.vocab;
        head.a.limit = c.logit_softcap;
        rk::dense(stream_, arith_, head, n_out, ws);
        prof_end(PC_HEAD, pt);
    }
}

int Engine::debug_keep_residual(bool on) {
    if (!stack_) {
        set_error("the residual stream is kept for layer-stack models only");
        return -1;
    }
    keep_residual_ = on;
    return 0;
}

int Engine::debug_read_residual(float * out, size_t n_floats, size_t * out_tokens) {
    if (!kept_residual_.ptr) {
        set_error("no step ran with the residual stream kept");
        return -1;
    }
    if (out_tokens) *out_tokens = (size_t)kept_tokens_;
    if (!out) return 0;
    const size_t per = (size_t)kept_tokens_ * stack_->width;
    if (n_floats < per * stack_runs_.size()) {
        set_error("the residual buffer is too small");
        return -2;
    }
    hip_check(hipStreamSynchronize(stream_), "debug_read_residual");
    for (size_t l = 0; l < stack_runs_.size(); ++l)
        hip_check(hipMemcpy(out + l * per, kept_residual_.as<float>() + l * (size_t)cfg_.n_batch * stack_->width, per * 4, hipMemcpyDeviceToHost), "hipMemcpy");
    return 0;
}

}  // namespace retro
