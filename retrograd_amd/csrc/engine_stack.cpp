// Layer-stack models in the engine: loading a checkpoint folder, the latent pools and recurrent state beside the paged
// cache, the step's plan for them and the forward pass. Slots, pages, packing, sampling, sequence operations and the
// generators are the engine's own (engine.cpp, generate.cpp).
#include "engine.hpp"
#include "safetensors_file.hpp"

#include <algorithm>
#include <cmath>
#include <cstring>

namespace retro {

namespace {

void hip_check(hipError_t err, const char * what) {
    if (err != hipSuccess) throw std::runtime_error(std::string("HIP error in ") + what + ": " + hipGetErrorString(err));
}

int up16(int n) { return (n + 15) / 16 * 16; }
int up32(int n) { return (n + 31) / 32 * 32; }

// Uploads a checkpoint's tensors and lays matrices out for the dense kernels.
class Loader {
public:
    Loader(const SafetensorsFile & f, hipStream_t s) : file_(f), stream_(s) {}

    void vector(const std::string & name, const std::vector<int64_t> & shape, DevBuf & out) {
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
        out.alloc(n * 4);
        hip_check(hipMemcpy(out.ptr, v.data(), n * 4, hipMemcpyHostToDevice), "hipMemcpy");
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
    // ... as rows row0 .. of m, its columns from k0 on.
    void matrix(const std::string & name, int rows, int cols, StackLayer::Matrix & m, int row0 = 0, int k0 = 0) {
        rk::dense_pack(stream_, raw(name, rows, cols), rows, cols, cols, 1, m.buf.as<uint16_t>(), m.w.kf, row0, k0);
    }
    void finish() { hip_check(hipStreamSynchronize(stream_), "hipStreamSynchronize"); }

private:
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
    hp_.n_layer = (int)c.layers.size();
    hp_.n_embd = c.width;
    hp_.n_vocab = c.vocab;
    hp_.eps = c.eps;
    const int E = c.width, KE = rk::frags_of(E);

    const StTensor & emb = file.require("embed", {c.vocab, E});
    if (emb.dtype != "BF16") throw std::runtime_error("tensor embed must be BF16");
    tok_embd_.w.type = rk::WT_BF16;
    tok_embd_.w.K = E;
    tok_embd_.w.N = c.vocab;
    tok_embd_.w.bytes = emb.nbytes;
    tok_embd_.buf.alloc(emb.nbytes);
    hip_check(hipMemcpy(tok_embd_.buf.ptr, emb.data, emb.nbytes, hipMemcpyHostToDevice), "hipMemcpy");
    tok_embd_.w.raw = tok_embd_.buf.as<uint8_t>();
    ld.shape(stack_head_, c.vocab, KE);
    ld.matrix("embed", c.vocab, E, stack_head_);
    ld.vector("final.norm", {E}, out_norm_);

    stack_layers_.resize(c.layers.size());
    for (size_t l = 0; l < c.layers.size(); ++l) {
        StackLayer & L = stack_layers_[l];
        L.spec = c.layers[l];
        const LayerSpec & sp = L.spec;
        const std::string p = "l" + std::to_string(l) + ".", m = p + "mix.";
        ld.vector(p + "norm1", {E}, L.norm);
        if (c.arch->layer_scale) {
            ld.vector(p + "ls1", {E}, L.scale_mix);
            if (sp.ff > 0) ld.vector(p + "ls2", {E}, L.scale_ff);
        }
        // input rows: the mixer's, in whole tiles, then the feed-forward's
        const LatentSpec & a = sp.latent;
        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            const bool own = a.kv_from < 0;
            L.kv_col = up16(a.q_rank);
            L.gate_col = L.kv_col + (own ? up16(a.kv_rank) : 0);
            L.in_rows = L.gate_col + a.heads;
            L.pool_layer = own ? (int)l : a.kv_from;
        } else {
            L.in_rows = sp.mamba.rows();
        }
        L.in_tiles = (L.in_rows + 15) / 16;
        ld.shape(L.w_in, sp.ff > 0 ? L.in_tiles * 16 + sp.ff : L.in_rows, KE);
        if (sp.ff > 0) ld.matrix(p + "mlp.up", sp.ff, E, L.w_in, L.in_tiles * 16);
        const int mix = sp.mix_width(), KM = rk::frags_of(mix);
        ld.shape(L.w_out, E, KM + (sp.ff > 0 ? rk::frags_of(sp.ff) : 0));
        ld.matrix(m + "o", E, mix, L.w_out);
        if (sp.ff > 0) ld.matrix(p + "mlp.down", E, sp.ff, L.w_out, 0, KM * 32);

        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            ld.matrix(m + "dq", a.q_rank, E, L.w_in);
            ld.vector(m + "dq.norm", {a.q_rank}, L.q_norm);
            if (a.kv_from < 0) {
                ld.matrix(m + "dkv", a.kv_rank, E, L.w_in, L.kv_col);
                ld.vector(m + "dkv.norm", {a.kv_rank}, L.kv_norm);
            }
            ld.matrix(m + "g", a.heads, E, L.w_in, L.gate_col);
            // queries head by head, every head padded to whole fragments
            const int D = up32(a.dim), R = 32 * rk::latent_frags(a.kv_rank);
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
        } else {
            const rk::MambaShape & s = sp.mamba;
            ld.matrix(m + "in", s.rows(), E, L.w_in);
            ld.vector(m + "conv", {s.channels(), s.taps}, L.conv_w);
            ld.vector(m + "conv.b", {s.channels()}, L.conv_b);
            ld.vector(m + "dt_bias", {s.heads}, L.dt_bias);
            ld.vector(m + "A_log", {s.heads}, L.A_log);
            ld.vector(m + "D", {s.heads}, L.D);
            ld.vector(m + "norm", {s.inner()}, L.gate_norm);
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

// Latent pools, recurrent state and the step's buffers.
void Engine::build_stack() {
    const StackConfig & c = *stack_;
    const size_t n_layer = c.layers.size(), elem = (size_t)arith_;
    const int B = (int)cfg_.n_batch, E = c.width, n_slots = (int)cfg_.n_seq_max;
    qt_ = 0;                                  // attention plans its own blocks
    k_pool_.resize(n_layer);
    v_pool_.resize(n_layer);
    size_t total = 0;
    std::vector<size_t> at(n_layer, 0), bytes(n_layer, 0);
    for (size_t l = 0; l < n_layer; ++l) {
        const LatentSpec & a = c.layers[l].latent;
        if (c.layers[l].mixer != Mixer::LATENT_ATTENTION || a.kv_from >= 0) continue;
        const int kf = rk::latent_frags(a.kv_rank);
        bytes[l] = (size_t)n_pages_ * rk::latent_page_elems(kf) * elem;
        at[l] = total;
        total += (bytes[l] + 255) / 256 * 256;
        cache_parts_.push_back({(int)l, false, (size_t)kf * 32 * elem});
    }
    kv_slab_.alloc(total);
    if (total) hip_check(hipMemsetAsync(kv_slab_.ptr, 0, total, stream_), "hipMemsetAsync");      // pages never hold non-finite values
    for (size_t l = 0; l < n_layer; ++l)
        if (bytes[l]) k_pool_[l] = PoolView{(uint8_t *)kv_slab_.ptr + at[l], bytes[l]};

    // recurrent state: [layer][slot] states, then two planes of [layer][slot] convolution inputs
    size_t states = 0;
    for (StackLayer & L : stack_layers_) {
        if (L.spec.mixer != Mixer::MAMBA2) continue;
        const rk::MambaShape & s = L.spec.mamba;
        L.state_slot = (size_t)s.heads * s.state * s.vdim;
        L.conv_slot = (size_t)(s.taps - 1) * s.channels();
        states += L.state_slot * n_slots;
        conv_plane_floats_ += L.conv_slot * n_slots;
        recurrent_slot_floats_ += L.state_slot + L.conv_slot;
    }
    recurrent_slab_.alloc((states + 2 * conv_plane_floats_) * 4);
    if (recurrent_slab_.ptr) {
        hip_check(hipMemsetAsync(recurrent_slab_.ptr, 0, recurrent_slab_.bytes, stream_), "hipMemsetAsync");
        float * st = recurrent_slab_.as<float>(), * cv = st + states;
        for (StackLayer & L : stack_layers_) {
            if (L.spec.mixer != Mixer::MAMBA2) continue;
            L.state = st;
            L.conv_state = cv;
            st += L.state_slot * n_slots;
            cv += L.conv_slot * n_slots;
        }
    }

    build_pack_buffers();
    build_step_buffers();
    const double magnitude = 1.0;             // no rotation: only the factor the packing kernel reads
    inv_freq_.alloc(sizeof(double));
    hip_check(hipMemcpy(inv_freq_.ptr, &magnitude, sizeof(double), hipMemcpyHostToDevice), "hipMemcpy");

    size_t h = rk::frag_elems(B, rk::frags_of(E)), cq = 0, q = 0, qa = 0, ol = 0, mix = 0, ff = 0, xbc = 0, y = 0;
    for (const LayerSpec & sp : c.layers) {
        mix = std::max(mix, rk::frag_elems(B, rk::frags_of(sp.mix_width())));
        if (sp.ff > 0) ff = std::max(ff, rk::frag_elems(B, rk::frags_of(sp.ff)));
        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            const LatentSpec & a = sp.latent;
            cq = std::max(cq, rk::frag_elems(B, rk::frags_of(a.q_rank)));
            q = std::max(q, rk::frag_elems(B, a.heads * rk::frags_of(a.dim)));
            qa = std::max(qa, (size_t)B * a.heads * 32 * rk::latent_frags(a.kv_rank));
            ol = std::max(ol, rk::frag_elems(B, a.heads * rk::latent_frags(a.kv_rank)));
        } else {
            xbc = std::max(xbc, (size_t)B * sp.mamba.channels());
            y = std::max(y, (size_t)B * sp.mamba.inner());
        }
    }
    for (const StackLayer & L : stack_layers_) st_proj_ld_ = std::max(st_proj_ld_, L.in_tiles * 16);
    auto zeroed = [&](DevBuf & b, size_t n) {       // padding that no producer writes has to be finite
        b.alloc(n);
        if (n) hip_check(hipMemsetAsync(b.ptr, 0, n, stream_), "hipMemsetAsync");
    };
    x_.alloc((size_t)B * E * 4);
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
    mm_ws_.alloc(rk::dense_workspace_floats() * 4);
}

// ---- recurrent state of a slot --------------------------------------------------------------------

void Engine::state_copy(int32_t src, int32_t dst) {
    const Slot & a = slots_[(size_t)src];
    Slot & b = slots_[(size_t)dst];
    b.plane = 0;
    for (const StackLayer & L : stack_layers_) {
        if (L.spec.mixer != Mixer::MAMBA2) continue;
        rk::copy_floats(stream_, L.state + src * L.state_slot, L.state + dst * L.state_slot, L.state_slot);
        rk::copy_floats(stream_, L.conv_state + a.plane * conv_plane_floats_ + src * L.conv_slot, L.conv_state + dst * L.conv_slot, L.conv_slot);
    }
}

void Engine::state_pack(int32_t slot, float * out) {
    const int plane = slots_[(size_t)slot].plane;
    auto get = [&](const float * src, size_t n) {
        if (n) hip_check(hipMemcpyAsync(out, src, n * 4, hipMemcpyDeviceToHost, stream_), "hipMemcpyAsync");
        out += n;
    };
    for (const StackLayer & L : stack_layers_) {
        if (L.spec.mixer != Mixer::MAMBA2) continue;
        get(L.state + slot * L.state_slot, L.state_slot);
        get(L.conv_state + plane * conv_plane_floats_ + slot * L.conv_slot, L.conv_slot);
    }
    hip_check(hipStreamSynchronize(stream_), "seq_save");
}

void Engine::state_unpack(int32_t slot, const float * in) {
    slots_[(size_t)slot].plane = 0;
    auto put = [&](float * dst, size_t n) {
        if (n) hip_check(hipMemcpyAsync(dst, in, n * 4, hipMemcpyHostToDevice, stream_), "hipMemcpyAsync");
        in += n;
    };
    for (const StackLayer & L : stack_layers_) {
        if (L.spec.mixer != Mixer::MAMBA2) continue;
        put(L.state + slot * L.state_slot, L.state_slot);
        put(L.conv_state + slot * L.conv_slot, L.conv_slot);
    }
    hip_check(hipStreamSynchronize(stream_), "seq_load");
}

// ---- the step's plan ------------------------------------------------------------------------------
// Blocks of query columns for every head count among the layers, and for recurrent models the tokens of every sequence
// in order (a step may hold several rows of one slot).

void Engine::plan_stack(const std::vector<RowView> & rows, const std::vector<std::pair<int, int>> & before) {
    block_plans_.clear();
    plan_blocks_.clear();
    plan_runs_.clear();
    plan_run_tok_.clear();
    plan_max_run_ = 0;
    step_rows_ = (int)rows.size();
    int total = 0;
    for (const RowView & r : rows) total += (int)r.n;
    for (const LayerSpec & sp : stack_->layers) {
        if (sp.mixer != Mixer::LATENT_ATTENTION) continue;
        const int H = sp.latent.heads, cols = rk::latent_block_cols(arith_, H, rk::latent_frags(sp.latent.kv_rank), total, (int)rows.size());
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
            s.plane = 1 - s.plane;            // this step leaves the convolution inputs in the other plane
            toks.emplace_back();
        }
        for (uint32_t i = 0; i < r.n; ++i) toks[(size_t)k].push_back(at + (int32_t)i);
        at += (int32_t)r.n;
    }
    for (size_t k = 0; k < plan_runs_.size(); ++k) {
        plan_runs_[k].start = (int32_t)plan_run_tok_.size();
        plan_runs_[k].n = (int32_t)toks[k].size();
        plan_max_run_ = std::max(plan_max_run_, plan_runs_[k].n);
        plan_run_tok_.insert(plan_run_tok_.end(), toks[k].begin(), toks[k].end());
    }
}

size_t Engine::stack_plan_bytes() const {
    return plan_runs_.size() * sizeof(rk::SeqRun) + plan_blocks_.size() * sizeof(rk::LatentBlock) + plan_run_tok_.size() * 4;
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
    d_blocks_ = (const rk::LatentBlock *)put(plan_blocks_.data(), plan_blocks_.size() * sizeof(rk::LatentBlock));
    d_run_tok_ = (const int32_t *)put(plan_run_tok_.data(), plan_run_tok_.size() * 4);
}

// ---- the forward pass -------------------------------------------------------------------------------

void Engine::forward_stack(int T, int n_out) {
    const StackConfig & c = *stack_;
    const int E = c.width, KE = rk::frags_of(E), ld = st_proj_ld_;
    float * x = x_.as<float>(), * proj = st_proj_.as<float>(), * ws = mm_ws_.as<float>();
    const rk::RowDesc * rows = d_stage_.as<rk::RowDesc>();
    rk::Slices pending;
    size_t pt = prof_begin(PC_EMBED);
    rk::embed(stream_, tok_embd_.w, pk_.tok, T, x);
    prof_end(PC_EMBED, pt);
    if (keep_residual_) {
        kept_residual_.ensure(stack_layers_.size() * (size_t)cfg_.n_batch * E * 4);
        kept_tokens_ = T;
    }
    for (size_t l = 0; l < stack_layers_.size(); ++l) {
        const StackLayer & L = stack_layers_[l];
        const LayerSpec & sp = L.spec;
        pt = prof_begin(PC_NORM);
        rk::norm_act(stream_, arith_, c.arch->norm, x, L.norm.as<float>(), E, c.eps, nullptr, T, st_h_.ptr, KE, pending);
        prof_end(PC_NORM, pt);
        pt = prof_begin(PC_QKV);
        rk::DenseJob in;
        in.w = L.w_in.w;
        in.x = {st_h_.ptr, KE, 0};
        in.split_tile = L.in_tiles;
        in.n_a = L.in_rows;
        in.a.kind = rk::OUT_F32; in.a.dst = proj; in.a.ld = ld;
        in.b.kind = c.arch->ff_act; in.b.dst = st_ff_.ptr; in.b.ld = rk::frags_of(std::max(sp.ff, 1));
        rk::dense(stream_, arith_, in, T, ws);
        prof_end(PC_QKV, pt);
        const int KM = rk::frags_of(sp.mix_width());
        if (sp.mixer == Mixer::LATENT_ATTENTION) {
            const LatentSpec & a = sp.latent;
            const int D = rk::frags_of(a.dim), R = rk::latent_frags(a.kv_rank), H = a.heads;
            pt = prof_begin(PC_ROPE);
            rk::LatentNorms n;
            n.proj = proj; n.ld = ld; n.q_rank = a.q_rank; n.kv_col = L.kv_col; n.kv_rank = a.kv_rank;
            n.q_w = L.q_norm.as<float>(); n.kv_w = L.kv_norm.as<float>(); n.eps = c.eps;
            n.act_q = st_cq_.ptr; n.act_q_kf = rk::frags_of(a.q_rank);
            n.pool = k_pool_[(size_t)L.pool_layer].ptr; n.pool_kf = R; n.cell = pk_.cell;
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
            pt = prof_begin(PC_ATTN);
            const BlockPlan * plan = nullptr;
            const int cols = rk::latent_block_cols(arith_, H, R, T, step_rows_);
            for (const BlockPlan & b : block_plans_) if (b.heads == H && b.cols == cols) plan = &b;
            rk::LatentAttn at;
            at.q = st_qa_.ptr; at.H = H; at.kf = R; at.window = a.window;
            at.rows = rows; at.blocks = d_blocks_ + plan->first; at.n_blocks = (int)plan->n; at.block_cols = plan->cols;
            at.table = table_.as<int32_t>(); at.max_pages = max_pages_;
            at.pool = k_pool_[(size_t)L.pool_layer].ptr;
            at.splits = rk::latent_splits(arith_, at, step_max_resident_);
            st_partial_.ensure(rk::latent_partial_floats(T, H, R, at.splits) * 4);
            at.partial_ml = st_partial_.as<float>();
            at.partial = at.partial_ml + (size_t)T * H * at.splits * 2;
            at.out = st_ol_.ptr; at.out_kf = H * R;
            rk::latent_attention(stream_, arith_, at);
            prof_end(PC_ATTN, pt);
            if (at.splits > 1) {
                pt = prof_begin(PC_COMBINE);
                rk::latent_combine(stream_, at, T);
                prof_end(PC_COMBINE, pt);
            }
            pt = prof_begin(PC_OPROJ);
            rk::DenseJob uv;
            uv.w = L.uv.w;
            uv.x = {st_ol_.ptr, H * R, R};
            uv.a.kind = rk::OUT_ACT_GATED; uv.a.dst = st_mix_.ptr; uv.a.ld = KM; uv.a.col_batch = a.vdim;
            uv.a.gate = proj + L.gate_col; uv.a.ld_gate = ld;
            rk::dense(stream_, arith_, uv, T, ws);
            prof_end(PC_OPROJ, pt);
        } else {
            pt = prof_begin(PC_SCAN);
            rk::MambaJob j;
            j.sh = sp.mamba;
            j.proj = proj; j.ld = ld;
            j.conv_w = L.conv_w.as<float>(); j.conv_b = L.conv_b.as<float>(); j.dt_bias = L.dt_bias.as<float>();
            j.A_log = L.A_log.as<float>(); j.D = L.D.as<float>(); j.norm_w = L.gate_norm.as<float>();
            j.eps = c.eps;
            j.runs = d_runs_; j.n_runs = (int)plan_runs_.size(); j.max_run = plan_max_run_; j.run_tok = d_run_tok_;
            j.conv_state = L.conv_state; j.conv_plane = conv_plane_floats_; j.state = L.state;
            j.xbc = st_xbc_.as<float>(); j.y = st_y_.as<float>();
            j.out = st_mix_.ptr; j.out_kf = KM;
            rk::mamba_mix(stream_, arith_, j, T);
            prof_end(PC_SCAN, pt);
        }
        pt = prof_begin(PC_DOWN);
        rk::DenseJob out;
        out.w = L.w_out.w;
        out.x = {st_mix_.ptr, KM, 0};
        out.kf1 = KM;
        out.scale1 = L.scale_mix.as<float>();
        if (sp.ff > 0) {
            out.x2 = {st_ff_.ptr, rk::frags_of(sp.ff), 0};
            out.scale2 = L.scale_ff.as<float>();
        }
        out.a.kind = rk::OUT_RESIDUAL; out.a.dst = x; out.a.ld = E;
        pending = rk::dense(stream_, arith_, out, T, ws);
        prof_end(PC_DOWN, pt);
        if (keep_residual_) {
            float * kept = kept_residual_.as<float>() + l * (size_t)cfg_.n_batch * E;
            rk::copy_floats(stream_, x, kept, (size_t)T * E);
            rk::add_slices(stream_, kept, E, T, pending);
        }
    }
    if (n_out > 0) {
        logits_.ensure((size_t)n_out * c.vocab * 4);
        pt = prof_begin(PC_HEAD);
        rk::norm_act(stream_, arith_, c.arch->norm, x, out_norm_.as<float>(), E, c.eps, pk_.out_tok, n_out, st_out_.ptr, KE, pending);
        rk::DenseJob head;
        head.w = stack_head_.w;
        head.x = {st_out_.ptr, KE, 0};
        head.a.kind = rk::OUT_F32; head.a.dst = logits_.ptr; head.a.ld = c.vocab;
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
    if (n_floats < per * stack_layers_.size()) {
        set_error("the residual buffer is too small");
        return -2;
    }
    hip_check(hipStreamSynchronize(stream_), "debug_read_residual");
    for (size_t l = 0; l < stack_layers_.size(); ++l)
        hip_check(hipMemcpy(out + l * per, kept_residual_.as<float>() + l * (size_t)cfg_.n_batch * stack_->width, per * 4, hipMemcpyDeviceToHost), "hipMemcpy");
    return 0;
}

}  // namespace retro
