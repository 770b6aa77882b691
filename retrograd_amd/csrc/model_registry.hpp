// The architectures this library runs and what tells them apart. GGUF architectures share one block (attention with
// rotation, SwiGLU or experts); layer-stack architectures come as a folder with config.json and model.safetensors, whose
// config lists every layer with its mixer and feed-forward.
#pragma once

#include "json_schema.hpp"
#include "stack_kernels.hpp"

#include <algorithm>
#include <cmath>
#include <fstream>
#include <sstream>
#include <stdexcept>
#include <string>
#include <vector>

#include <sys/stat.h>

namespace retro {

struct GgufArch { const char * name; bool rope_neox; };
inline const GgufArch * find_gguf_arch(const std::string & name) {
    static const GgufArch known[] = {{"llama", false}, {"qwen2", true}, {"qwen3", true}, {"qwen3moe", true}};
    for (const GgufArch & a : known) if (name == a.name) return &a;
    return nullptr;
}

// What an architecture fixes about its layers. Parallel layers: x <- x + scale1 * mixer(n(x)) + scale2 * ff(n(x)), one
// norm for both; otherwise x <- x + mixer(n1(x)), then x <- x + ff(n2(x)), and with norms after a
// sublayer x <- x + mult * n1b(mixer(n1(x))), and so on. The norm's kind and whether its weights are stored as differences from
// one; the activations (DenseOut kinds) of the feed-forward and of experts; element-wise
// layer scales or none; whether a dense feed-forward has biases, a shared expert a gate per token, and the head its own matrix.
// Grouped attention: what positions a mask of some size leaves; whether the values are the keys before rotation or a
// projection of their own, with biases on all three; how a head's columns pair up for rotation (i with i + dims / 2, or
// neighbours) and what stretching the rotation means; whether queries and keys are normed over all their heads before it, and
// whether the output has a bias too.
enum class Mask { WINDOW, CHUNK };
enum class Stretch { RAMP, BANDS };
enum class Pairs { HALVES, NEIGHBOURS };
struct StackArch {
    const char * name;
    int norm;
    bool norm_around_one, parallel;
    int ff_act, expert_act;
    bool layer_scale, ff_bias, shared_gate, own_head;
    Mask mask;
    bool keys_are_values;
    Pairs pairs;
    Stretch stretch;
    int score;                   // what an expert's weight is (rk::SCORE_*)
    bool qk_norm, out_bias;
    bool norm_after;             // norms after the sublayers, and of the embedding, to which one of two neighbouring tokens is added
    bool weigh_input;            // an expert's weight multiplies what it reads
    // Queries, keys and values leave the input product's epilogue for their places (norms over all heads need the whole row first).
    bool rows_in_place() const { return keys_are_values || !qk_norm; }
};
inline const StackArch * find_stack_arch(const std::string & name) {
    static const StackArch known[] = {
        {"Dibosun", rk::NORM_LAYER, false, true, rk::OUT_ACT_RELU2, -1, true, false, true, false, Mask::WINDOW, true, Pairs::HALVES, Stretch::RAMP, rk::SCORE_OVER_CHOSEN, false, false, false, false},
        {"Pomisun", rk::NORM_RMS, true, false, rk::OUT_ACT_GEGLU, rk::OUT_ACT_SWIGLU, false, false, true, false, Mask::CHUNK, true, Pairs::HALVES, Stretch::RAMP, rk::SCORE_OVER_CHOSEN, false, false, false, false},
        {"Vifanex", rk::NORM_RMS, false, false, rk::OUT_ACT_CLAMPED, rk::OUT_ACT_CLAMPED, false, true, false, true, Mask::WINDOW, false, Pairs::NEIGHBOURS, Stretch::BANDS, rk::SCORE_OVER_ALL, true, false, false, false},
        {"Kilurax", rk::NORM_RMS, false, false, rk::OUT_ACT_SWIGLU, rk::OUT_ACT_SWIGLU, false, false, false, true, Mask::WINDOW, false, Pairs::HALVES, Stretch::RAMP, rk::SCORE_SIGMOID, false, true, true, true},
    };
    for (const StackArch & a : known) if (name == a.name) return &a;
    return nullptr;
}

// DELTA: every mixer with a matrix state and a rule of writing (its DeltaShape says which). ATTENTION_MAMBA2: both over one input,
// their outputs scaled and added.
enum class Mixer { LATENT_ATTENTION, MAMBA2, ATTENTION, DELTA, ATTENTION_MAMBA2 };

struct LatentSpec {
    int heads = 0, dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;
    int window = 0;              // 0: every earlier position is seen
    int kv_from = -1;            // the layer whose latents are attended to (-1: this layer's own)
    float scale = 1.0f;
};

// Rotary positions on the first `dims` columns of a head, optionally stretched: frequencies that turn fewer than `slow` times
// within the original length are divided by the factor, those above `fast` kept. In between a ramp over the index of the
// pair, which also lengthens the rotated vectors (RAMP, as in YaRN), or one over the number of turns (BANDS, as in Llama 3.1).
struct RotarySpec {
    int dims = 0;
    double base = 10000.0, factor = 1.0, original = 0.0, fast = 0.0, slow = 0.0;      // original 0: not stretched
    Stretch stretch = Stretch::RAMP;
    bool operator==(const RotarySpec & o) const {
        return dims == o.dims && stretch == o.stretch && base == o.base && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
    // Radians per position of the dims / 2 pairs.
    std::vector<double> frequencies() const {
        std::vector<double> f((size_t)(dims / 2));
        const double pi = 3.14159265358979323846;
        auto pair_of = [&](double turns) { return dims * std::log(original / (2.0 * pi * turns)) / (2.0 * std::log(base)); };
        const double lo = original > 0.0 ? std::max(std::floor(pair_of(fast)), 0.0) : 0.0;
        const double hi = original > 0.0 ? std::min(std::ceil(pair_of(slow)), dims - 1.0) : 0.0;
        for (size_t i = 0; i < f.size(); ++i) {
            f[i] = std::pow(base, -2.0 * (double)i / dims);
            if (original <= 0.0) continue;
            if (stretch == Stretch::BANDS) {
                const double turns = original * f[i] / (2.0 * pi);
                const double keep = turns > fast ? 1.0 : turns < slow ? 0.0 : fast > slow ? (turns - slow) / (fast - slow) : 1.0;
                f[i] = keep * f[i] + (1.0 - keep) * f[i] / factor;
                continue;
            }
            const double ramp = std::min(std::max(((double)i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp);
        }
        return f;
    }
    double magnitude() const { return original > 0.0 && stretch == Stretch::RAMP ? 0.1 * std::log(factor) + 1.0 : 1.0; }      // of cosines and sines
};

// Grouped attention. Layers that mix their values take a share of those of the first such layer (of the same token).
struct AttentionSpec {
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    bool v_mix = false, v_first = false;
    rk::PairFrags frags() const { return dim == vdim ? rk::PairFrags{rk::cache_frags(dim), rk::cache_frags(dim)} : rk::pair_frags(dim, vdim); }
    int window = 0, chunk = 0;   // positions seen: the last `window`, or those of the same chunk (0: no bound)
    float scale = 1.0f, softcap = 0.0f;
    RotarySpec rot;
};

// Experts of a feed-forward: every token takes `top` of them, out of the `keep` best of `groups` groups of neighbours, and
// the shared one (ff 0: none). The limits are those of clamped activations.
struct MoeSpec {
    int experts = 0, top = 0, ff = 0, shared_ff = 0, groups = 1, keep = 1;
    float limit = 0.0f, shared_limit = 0.0f, scale = 1.0f;
};

struct LayerSpec {
    Mixer mixer = Mixer::LATENT_ATTENTION;
    LatentSpec latent;
    rk::MambaShape mamba;
    AttentionSpec attention;
    rk::DeltaShape delta;
    float left_scale = 1.0f, right_scale = 1.0f;      // of attention and Mamba-2 side by side
    int ff = 0;                  // of a dense feed-forward; 0 and no experts: no feed-forward
    float ff_limit = 0.0f;
    MoeSpec moe;
    bool has_ff() const { return ff > 0 || moe.experts > 0; }
    bool grouped_attention() const { return mixer == Mixer::ATTENTION || mixer == Mixer::ATTENTION_MAMBA2; }
    bool state_space() const { return mixer == Mixer::MAMBA2 || mixer == Mixer::ATTENTION_MAMBA2; }
    bool attends() const { return mixer == Mixer::LATENT_ATTENTION || grouped_attention(); }
    bool recurrent() const { return state_space() || mixer == Mixer::DELTA; }
    // Columns a mixer hands to its output projection (a head of grouped attention padded as its cached values are), and those of
    // Mamba-2 beside attention.
    int beside_width() const { return mixer == Mixer::ATTENTION_MAMBA2 ? mamba.inner() : 0; }
    int mix_width() const {
        switch (mixer) {
            case Mixer::MAMBA2: return mamba.inner();
            case Mixer::DELTA: return delta.inner();
            case Mixer::ATTENTION:
            case Mixer::ATTENTION_MAMBA2: return attention.heads * 32 * attention.frags().v;
            default: return latent.heads * latent.vdim;
        }
    }
};

// One pass through a layer; a looped layer has several, each with its own cache or state.
struct LayerRun { int layer; bool add_embedding; };      // the embedding output is added to the stream first

struct StackConfig {
    const StackArch * arch = nullptr;
    int width = 0, vocab = 0;
    float eps = 0.0f;
    float embedding_scale = 1.0f, logit_softcap = 0.0f;      // 0: none
    int streams = 0;             // residual streams of hyper-connections (0: a plain residual sum)
    int norm_groups = 1;         // equal parts of a row, normed each by its own
    float residual_mult = 1.0f;  // of what a sublayer adds
    int input_taps = 0;          // of the convolution over the tokens that every sublayer's input goes through (0: none)
    int64_t pair_buckets = 0, pair_mul_prev = 0, pair_mul_cur = 0;      // an embedding of every two neighbouring tokens 
    // The sublayers' norms are k_sublayer_norm's.
    bool around() const { return arch->norm_after || norm_groups > 1 || residual_mult != 1.0f || input_taps > 0; }
    std::vector<LayerSpec> layers;
    std::vector<LayerRun> runs;
    bool recurrent() const {
        for (const LayerSpec & l : layers) if (l.recurrent()) return true;
        return input_taps > 0 || pair_buckets > 0;
    }

    static bool is_folder(const std::string & path) {
        struct stat st {};
        return ::stat(path.c_str(), &st) == 0 && S_ISDIR(st.st_mode);
    }
    static StackConfig read(const std::string & folder) {
        std::ifstream in(folder + "/config.json", std::ios::binary);
        if (!in) throw std::runtime_error("cannot open " + folder + "/config.json");
        std::stringstream text;
        text << in.rdbuf();
        return parse(JsonParser::parse(text.str()));
    }
    static StackConfig parse(const JsonValue & v) {
        StackConfig c;
        const JsonValue & name = need(v, "architecture");
        c.arch = find_stack_arch(name.text);
        if (!c.arch) throw std::runtime_error("unsupported model architecture: " + name.text);
        c.width = size(v, "width");
        c.vocab = size(v, "vocab");
        c.eps = (float)number(need(v, "norm"), "eps");
        if (present(v, "embedding") && present(need(v, "embedding"), "scale")) c.embedding_scale = (float)number(need(v, "embedding"), "scale");
        if (present(v, "logit_softcap")) c.logit_softcap = (float)number(v, "logit_softcap");
        if (!(c.logit_softcap >= 0.0f)) throw std::runtime_error("config.json: 'logit_softcap' must not be negative");
        if (present(v, "streams")) c.streams = size(v, "streams");
        if (c.streams > rk::MAX_STREAMS || (c.streams > 0 && (c.arch->parallel || c.arch->norm != rk::NORM_RMS || present(v, "loop"))))
            throw std::runtime_error("config.json: 'streams' of sequential layers over RMS norms, without a loop, " + std::to_string(rk::MAX_STREAMS) + " at most");
        const JsonValue & norm = need(v, "norm");
        if (present(norm, "groups")) c.norm_groups = size(norm, "groups");
        if (c.width % c.norm_groups != 0) throw std::runtime_error("config.json: 'width' must be a multiple of 'norm.groups'");
        if (present(v, "residual_mult")) c.residual_mult = (float)number(v, "residual_mult");
        if (present(v, "canon")) c.input_taps = size(need(v, "canon"), "taps");
        if (c.arch->norm_after) {
            const JsonValue & b = need(need(v, "embedding"), "bigram");
            c.pair_buckets = size(b, "buckets");
            c.pair_mul_prev = factor(b, "mul_prev") % c.pair_buckets;      // of residues the products fit 64 bits
            c.pair_mul_cur = factor(b, "mul_cur") % c.pair_buckets;
        }
        if (c.around() && (c.arch->parallel || c.arch->norm != rk::NORM_RMS || c.streams > 0 || present(v, "loop")))
            throw std::runtime_error("config.json: grouped norms, 'residual_mult' and 'canon' need sequential layers over RMS norms, without streams or a loop");
        for (const JsonValue & l : need(v, "layers").items) c.layers.push_back(layer(*c.arch, l, c.layers));
        const int n = (int)c.layers.size();
        if (n < 1 || n > 4096) throw std::runtime_error("config.json: 'layers' must list 1 to 4096 layers");
        int start = 0, stop = 0, times = 1;
        if (present(v, "loop")) {
            const JsonValue & l = need(v, "loop");
            start = size(l, "start", 0);
            stop = size(l, "stop", 0);
            times = size(l, "times");
            if (start > stop || stop > n || (int64_t)(stop - start) * times > 65536) throw std::runtime_error("config.json: 'loop' must name a range of layers");
        }
        for (int l = 0; l < start; ++l) c.runs.push_back({l, false});
        for (int t = 0; t < times; ++t)
            for (int l = start; l < stop; ++l) c.runs.push_back({l, t > 0 && l == start});
        for (int l = stop; l < n; ++l) c.runs.push_back({l, false});
        return c;
    }

private:
    static const JsonValue & need(const JsonValue & v, const char * key) {
        const JsonValue * m = v.get(key);
        if (!m) throw std::runtime_error(std::string("config.json lacks '") + key + "'");
        return *m;
    }
    static double number(const JsonValue & v, const char * key) {
        const JsonValue & m = need(v, key);
        if (m.kind != JsonValue::NUMBER) throw std::runtime_error(std::string("config.json: '") + key + "' must be a number");
        return m.num;
    }
    static int size(const JsonValue & v, const char * key, int lo = 1) {
        const double n = number(v, key);
        if (n < lo || n > (1 << 24) || n != (double)(int)n) throw std::runtime_error(std::string("config.json: '") + key + "' is no size");
        return (int)n;
    }
    static int64_t factor(const JsonValue & v, const char * key) {
        const double n = number(v, key);
        if (!(n >= 0.0) || n > 9007199254740992.0 || n != std::floor(n)) throw std::runtime_error(std::string("config.json: '") + key + "' is no whole number");
        return (int64_t)n;
    }
    static bool present(const JsonValue & v, const char * key) {
        const JsonValue * m = v.get(key);
        return m && m->kind != JsonValue::NUL;
    }
    static bool positive(double v) { return v > 0.0 && std::isfinite(v); }
    static float limit(const StackArch & arch, int act, const JsonValue & v) {
        if (act != rk::OUT_ACT_CLAMPED) return 0.0f;
        const double l = number(v, "limit");
        if (!(l > 0.0)) throw std::runtime_error("config.json: 'limit' must be positive");
        return (float)l;
    }
    static RotarySpec rotary(const StackArch & arch, const JsonValue & v, int dim) {
        RotarySpec r;
        r.stretch = arch.stretch;
        r.dims = size(v, "dims", 0);
        r.base = number(v, "base");
        if (r.dims > dim || r.dims % 2 != 0) throw std::runtime_error("config.json: 'rot.dims' must be even and within a head");
        if (!positive(r.base) || r.base == 1.0) throw std::runtime_error("config.json: 'rot.base' must be positive and not 1");
        if (present(v, "scaling")) {
            const JsonValue & s = need(v, "scaling");
            r.factor = number(s, "factor");
            r.original = number(s, "original");
            r.fast = number(s, arch.stretch == Stretch::BANDS ? "high" : "fast");
            r.slow = number(s, arch.stretch == Stretch::BANDS ? "low" : "slow");
            if (!positive(r.factor) || !positive(r.original) || !positive(r.fast) || !positive(r.slow))
                throw std::runtime_error("config.json: 'rot.scaling' must hold positive numbers");
        }
        return r;
    }
    static rk::MambaShape mamba2(const JsonValue & m) {
        rk::MambaShape s;
        s.heads = size(m, "heads");
        s.vdim = size(m, "vdim");
        s.state = size(m, "state");
        s.groups = size(m, "groups");
        s.taps = size(m, "conv");
        s.norm_groups = size(m, "norm_groups");
        if (s.heads % s.groups != 0) throw std::runtime_error("mamba2: heads must be a multiple of groups");
        if (s.inner() % s.norm_groups != 0) throw std::runtime_error("mamba2: heads * vdim must be a multiple of norm_groups");
        if (s.state > 512) throw std::runtime_error("mamba2: a state above 512 rows is not supported");
        return s;
    }
    static AttentionSpec attention(const StackArch & arch, const JsonValue & m, const std::vector<LayerSpec> & before) {
        AttentionSpec a;
        a.heads = size(m, "heads");
        a.kv_heads = size(m, "kv_heads");
        a.dim = size(m, "dim");
        a.scale = (float)number(m, "scale");
        if (present(m, "softcap")) a.softcap = (float)number(m, "softcap");
        if (present(m, "mask") && present(need(m, "mask"), "size")) (arch.mask == Mask::CHUNK ? a.chunk : a.window) = size(need(m, "mask"), "size");
        if (a.heads % a.kv_heads != 0) throw std::runtime_error("attention: heads must be a multiple of kv_heads");
        a.vdim = size(m, "vdim");
        if (arch.keys_are_values && a.vdim != a.dim) throw std::runtime_error("attention: the values are the keys, so vdim must be dim");
        if (a.dim > 1024 || a.vdim > 1024) throw std::runtime_error("attention: heads above 1024 columns are not supported");
        if (!arch.rows_in_place() && present(m, "v_mix")) a.v_mix = need(m, "v_mix").b;
        a.v_first = a.v_mix;
        for (const LayerSpec & b : before)
            if (b.mixer == Mixer::ATTENTION && b.attention.v_mix) {
                a.v_first = false;
                if (a.v_mix && b.attention.kv_heads * b.attention.vdim != a.kv_heads * a.vdim)
                    throw std::runtime_error("attention: layers that mix their values must have equally many");
            }
        if (!(a.softcap >= 0.0f)) throw std::runtime_error("attention: softcap must not be negative");
        if (arch.keys_are_values || present(m, "rot")) a.rot = rotary(arch, need(m, "rot"), a.dim);
        return a;
    }
    static rk::DeltaShape delta(const JsonValue & m, const std::string & type) {
        rk::DeltaShape s;
        s.heads = size(m, "heads");
        s.kv_heads = size(m, "kv_heads");
        s.dim = size(m, "dim");
        s.vdim = size(m, "vdim");
        s.taps = size(m, "conv");
        if (s.heads % s.kv_heads != 0) throw std::runtime_error(type + ": heads must be a multiple of kv_heads");
        state_limits(s, type);
        return s;
    }
    static void state_limits(const rk::DeltaShape & s, const std::string & type) {
        if (s.dim > 512 || s.vdim > 4096) throw std::runtime_error(type + ": at most 512 key and 4096 value channels per head are supported");
    }
    static LayerSpec layer(const StackArch & arch, const JsonValue & v, const std::vector<LayerSpec> & before) {
        LayerSpec l;
        const std::string type = need(v, "type").text;
        const JsonValue & m = need(v, "mixer");
        if (type == "latent_attention") {
            LatentSpec & a = l.latent;
            a.heads = size(m, "heads");
            a.dim = size(m, "dim");
            a.vdim = size(m, "vdim");
            a.q_rank = size(m, "q_rank");
            a.kv_rank = size(m, "kv_rank");
            a.scale = (float)number(m, "scale");
            if (present(m, "mask") && present(need(m, "mask"), "size")) a.window = size(need(m, "mask"), "size");
            if (present(m, "kv_from")) {
                a.kv_from = size(m, "kv_from", 0);
                if (a.kv_from >= (int)before.size() || before[(size_t)a.kv_from].mixer != Mixer::LATENT_ATTENTION
                        || before[(size_t)a.kv_from].latent.kv_from >= 0 || before[(size_t)a.kv_from].latent.kv_rank != a.kv_rank)
                    throw std::runtime_error("config.json: 'kv_from' must name an earlier latent attention layer with latents of its own and the same kv_rank");
            }
            if (a.kv_rank > 1024) throw std::runtime_error("latent attention: kv_rank above 1024 is not supported");
        } else if (type == "mamba2") {
            l.mixer = Mixer::MAMBA2;
            l.mamba = mamba2(m);
        } else if (type == "attention") {
            l.mixer = Mixer::ATTENTION;
            l.attention = attention(arch, m, before);
        } else if (type == "parallel") {
            if (arch.keys_are_values || arch.qk_norm || arch.parallel) throw std::runtime_error("config.json: 'parallel' mixers are not supported for this architecture");
            l.mixer = Mixer::ATTENTION_MAMBA2;
            l.attention = attention(arch, need(m, "left"), before);
            l.mamba = mamba2(need(m, "right"));
            l.left_scale = (float)number(m, "left_scale");
            l.right_scale = (float)number(m, "right_scale");
        } else if (type == "hgrn2") {
            l.mixer = Mixer::DELTA;
            rk::DeltaShape & s = l.delta;
            s.rule = rk::RULE_FORGET;
            s.gate = rk::GATE_NONE;
            s.heads = s.kv_heads = size(m, "heads");
            s.dim = size(m, "dim");
            s.vdim = size(m, "vdim");
            state_limits(s, type);
        } else if (type == "delta") {
            l.mixer = Mixer::DELTA;
            l.delta = delta(m, type);
            l.delta.rule = rk::RULE_DELTA_HEADS;
            l.delta.gate = rk::GATE_SILU;
        } else if (type == "channel_delta") {
            l.mixer = Mixer::DELTA;
            l.delta = delta(m, type);
        } else {
            throw std::runtime_error("config.json: unknown layer type '" + type + "'");
        }
        if (present(v, "mlp")) {
            const JsonValue & f = need(v, "mlp");
            const std::string kind = need(f, "kind").text;
            if (kind == "dense") {
                l.ff = size(f, "ff");
                l.ff_limit = limit(arch, arch.ff_act, f);
            } else if (kind == "moe" && arch.expert_act >= 0) {
                const JsonValue & r = need(f, "router");
                l.moe.experts = size(r, "experts");
                l.moe.top = size(r, "top");
                l.moe.ff = size(need(f, "expert"), "ff");
                l.moe.limit = limit(arch, arch.expert_act, need(f, "expert"));
                if (present(f, "shared")) {
                    l.moe.shared_ff = size(need(f, "shared"), "ff");
                    l.moe.shared_limit = limit(arch, arch.expert_act, need(f, "shared"));
                }
                if (present(r, "scale")) l.moe.scale = (float)number(r, "scale");
                if (present(r, "groups")) {
                    l.moe.groups = size(need(r, "groups"), "count");
                    l.moe.keep = size(need(r, "groups"), "keep");
                    if (l.moe.experts % l.moe.groups != 0 || l.moe.keep > l.moe.groups || l.moe.keep * (l.moe.experts / l.moe.groups) < l.moe.top)
                        throw std::runtime_error("moe: 'groups' must be equal parts of the experts, of which those kept hold at least 'top'");
                }
                if (l.moe.top > l.moe.experts) throw std::runtime_error("moe: 'top' exceeds 'experts'");
                if (l.moe.experts > rk::MAX_EXPERTS || l.moe.top > rk::MAX_TOP) throw std::runtime_error("moe: more experts than are supported");
            } else {
                throw std::runtime_error("config.json: unknown feed-forward kind '" + kind + "'");
            }
        }
        return l;
    }
};

}  // namespace retro
