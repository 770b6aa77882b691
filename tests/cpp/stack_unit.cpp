// Reads a checkpoint folder's config.json and model.safetensors with the engine's readers and prints what they found, or
// the refusal. Built and driven by tests/test_stack_files.py; CPU only.
#include <cstdio>
#include <exception>

#include "../../retrograd_amd/csrc/model_registry.hpp"
#include "../../retrograd_amd/csrc/safetensors_file.hpp"

int main(int argc, char ** argv) {
    if (argc != 3) return 2;
    const std::string folder = argv[1], what = argv[2];
    try {
        if (what == "config") {
            const retro::StackConfig c = retro::StackConfig::read(folder);
            std::printf("%s width %d vocab %d eps %g\n", c.arch->name, c.width, c.vocab, (double)c.eps);
            if (c.runs.size() != c.layers.size()) {
                std::printf("runs");
                for (const retro::LayerRun & r : c.runs) std::printf(" %s%d", r.add_embedding ? "+" : "", r.layer);
                std::printf("\n");
            }
            if (c.streams > 0) std::printf("streams %d embedding_scale %g logit_softcap %g\n", c.streams, (double)c.embedding_scale, (double)c.logit_softcap);
            if (c.around())
                std::printf("embedding_scale %g buckets %lld factors %lld %lld norm groups %d residual %g taps %d\n", (double)c.embedding_scale, (long long)c.pair_buckets,
                            (long long)c.pair_mul_prev, (long long)c.pair_mul_cur, c.norm_groups, (double)c.residual_mult, c.input_taps);
            for (const retro::LayerSpec & l : c.layers) {
                if (c.streams > 0) {
                    const retro::MoeSpec & e = l.moe;
                    std::printf("limits %g %g %g groups %d keep %d scale %g vdim %d v_mix %d v_first %d\n", (double)l.ff_limit, (double)e.limit, (double)e.shared_limit,
                                e.groups, e.keep, (double)e.scale, l.attention.vdim, l.attention.v_mix, l.attention.v_first);
                }
                if (l.mixer == retro::Mixer::ATTENTION_MAMBA2) {
                    const retro::AttentionSpec & g = l.attention;
                    const rk::MambaShape & s = l.mamba;
                    std::printf("parallel heads %d kv_heads %d dim %d vdim %d rot %d base %g scale %g times %g, heads %d vdim %d state %d groups %d taps %d norm_groups %d times %g, "
                                "ff %d experts %d top %d of %d shared %d\n", g.heads, g.kv_heads, g.dim, g.vdim, g.rot.dims, g.rot.base, (double)g.scale, (double)l.left_scale,
                                s.heads, s.vdim, s.state, s.groups, s.taps, s.norm_groups, (double)l.right_scale, l.ff, l.moe.experts, l.moe.top, l.moe.ff, l.moe.shared_ff);
                    continue;
                }
                if (l.mixer == retro::Mixer::DELTA) {
                    const rk::DeltaShape & d = l.delta;
                    const char * names[] = {"channel_delta", "delta", "hgrn2"};
                    std::printf("%s heads %d kv_heads %d dim %d vdim %d taps %d ff %d experts %d top %d of %d shared %d\n", names[d.rule], d.heads, d.kv_heads, d.dim, d.vdim,
                                d.taps, l.ff, l.moe.experts, l.moe.top, l.moe.ff, l.moe.shared_ff);
                    continue;
                }
                if (l.mixer == retro::Mixer::ATTENTION) {
                    const retro::AttentionSpec & g = l.attention;
                    std::printf("attention heads %d kv_heads %d dim %d window %d chunk %d scale %g softcap %g ff %d experts %d top %d of %d shared %d\n", g.heads, g.kv_heads,
                                g.dim, g.window, g.chunk, (double)g.scale, (double)g.softcap, l.ff, l.moe.experts, l.moe.top, l.moe.ff, l.moe.shared_ff);
                    std::printf("rotary %d magnitude %.17g", g.rot.dims, g.rot.magnitude());
                    for (double f : g.rot.frequencies()) std::printf(" %.17g", f);
                    std::printf("\n");
                    continue;
                }
                const retro::LatentSpec & a = l.latent;
                const rk::MambaShape & s = l.mamba;
                if (l.mixer == retro::Mixer::MAMBA2)
                    std::printf("mamba2 heads %d vdim %d state %d groups %d taps %d norm_groups %d ff %d\n", s.heads, s.vdim, s.state, s.groups, s.taps, s.norm_groups, l.ff);
                else
                    std::printf("latent heads %d dim %d vdim %d q_rank %d kv_rank %d window %d from %d scale %g ff %d\n", a.heads, a.dim, a.vdim, a.q_rank, a.kv_rank,
                                a.window, a.kv_from, (double)a.scale, l.ff);
            }
        } else {
            retro::SafetensorsFile f(folder + "/model.safetensors");
            const retro::StTensor * t = f.find(what);
            std::printf("%llu bytes, %s %s\n", (unsigned long long)f.tensor_bytes(), what.c_str(), t ? t->dtype.c_str() : "missing");
        }
        return 0;
    } catch (const std::exception & e) {
        std::printf("refused: %s\n", e.what());
        return 1;
    }
}
