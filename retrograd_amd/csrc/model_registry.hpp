// The architectures this library runs and what tells them apart. GGUF architectures share one block (attention with
// rotation, SwiGLU or experts); layer-stack architectures come as a folder with config.json and model.safetensors, whose
// config lists every layer with its mixer and feed-forward.
#pragma once

#include "json_schema.hpp"
#include "stack_kernels.hpp"

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

// What an architecture fixes about its layers: x <- x + scale1 * mixer(norm(x)) + scale2 * ff(norm(x)), one norm for
// both; the norm's kind, the feed-forward's activation (a DenseOut kind), element-wise layer scales or none.
struct StackArch { const char * name; int norm; int ff_act; bool layer_scale; };
inline const StackArch * find_stack_arch(const std::string & name) {
    static const StackArch known[] = {{"Dibosun", rk::NORM_LAYER, rk::OUT_ACT_RELU2, true}};
    for (const StackArch & a : known) if (name == a.name) return &a;
    return nullptr;
}

enum class Mixer { LATENT_ATTENTION, MAMBA2 };

struct LatentSpec {
    int heads = 0, dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;
    int window = 0;              // 0: every earlier position is seen
    int kv_from = -1;            // the layer whose latents are attended to (-1: this layer's own)
    float scale = 1.0f;
};

struct LayerSpec {
    Mixer mixer = Mixer::LATENT_ATTENTION;
    LatentSpec latent;
    rk::MambaShape mamba;
    int ff = 0;                  // 0: no feed-forward
    int mix_width() const { return mixer == Mixer::MAMBA2 ? mamba.inner() : latent.heads * latent.vdim; }
};

struct StackConfig {
    const StackArch * arch = nullptr;
    int width = 0, vocab = 0;
    float eps = 0.0f;
    std::vector<LayerSpec> layers;
    bool recurrent() const {
        for (const LayerSpec & l : layers) if (l.mixer == Mixer::MAMBA2) return true;
        return false;
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
        for (const JsonValue & l : need(v, "layers").items) c.layers.push_back(layer(l, c.layers));
        if (c.layers.empty() || c.layers.size() > 4096) throw std::runtime_error("config.json: 'layers' must list 1 to 4096 layers");
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
    static bool present(const JsonValue & v, const char * key) {
        const JsonValue * m = v.get(key);
        return m && m->kind != JsonValue::NUL;
    }
    static LayerSpec layer(const JsonValue & v, const std::vector<LayerSpec> & before) {
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
            rk::MambaShape & s = l.mamba;
            s.heads = size(m, "heads");
            s.vdim = size(m, "vdim");
            s.state = size(m, "state");
            s.groups = size(m, "groups");
            s.taps = size(m, "conv");
            s.norm_groups = size(m, "norm_groups");
            if (s.heads % s.groups != 0) throw std::runtime_error("mamba2: heads must be a multiple of groups");
            if (s.inner() % s.norm_groups != 0) throw std::runtime_error("mamba2: heads * vdim must be a multiple of norm_groups");
            if (s.state > 512) throw std::runtime_error("mamba2: a state above 512 rows is not supported");
        } else {
            throw std::runtime_error("config.json: unknown layer type '" + type + "'");
        }
        if (present(v, "mlp")) {
            const JsonValue & f = need(v, "mlp");
            const std::string kind = need(f, "kind").text;
            if (kind != "dense") throw std::runtime_error("config.json: unknown feed-forward kind '" + kind + "'");
            l.ff = size(f, "ff");
        }
        return l;
    }
};

}  // namespace retro
