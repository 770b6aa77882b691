"""Prefill and decode of layer-stack models at sizes that resemble a real model's layers, beside the closest other models of
the same width, feed-forward width and depth: what `bench.py --model dibosun`, `--model pomisun`, `--model vifanex` and `--model kilurax` run. Weights are random
(seeded), prompts random token ids. Every kernel category is also priced against its roofline, the larger of its
algorithmic bytes over 8 TB/s and its products' flops over 2.5 PFLOP/s (a product counted once, however a model's
arithmetic splits its operands; the scan's flops over the 157 TFLOP/s of f32)."""

from __future__ import annotations

import json
import os
import sys
import time
from pathlib import Path

import numpy as np

HBM, BF16, F32 = 8e12, 2.5e15, 157e12
N_SEQ_MAX, CONTEXT = 64, 1024

# width, feed-forward, heads, dim, q_rank, kv_rank, mamba heads (of 64 x 128 state), groups
SIZES = {"w2048": (2048, 8192, 16, 128, 768, 512, 64, 8), "w4096": (4096, 14336, 32, 128, 1536, 512, 128, 8)}
VOCAB, WINDOW, CHUNK = 32000, 1024, 2048
# experts, experts per token, their width, the shared expert's
EXPERTS = {"w2048": (64, 8, 768, 1536), "w4096": (32, 4, 1536, 3072)}


def dibosun_config(size):
    from . import synth_stack as Y
    E, F, H, D, QR, R, MH, G = SIZES[size]
    lat = lambda kv_from=None: Y.latent_layer(H, D, D, QR, R, WINDOW, F, kv_from=kv_from)
    mam = lambda: Y.mamba2_layer(MH, 64, 128, G, 4, G, F)
    return Y.dibosun(E, VOCAB, [lat(), mam(), lat(0), mam(), lat(), mam(), lat(4), mam()])


def pomisun_config(size):
    from . import synth_stack as Y
    E, F, H, D = SIZES[size][:4]
    layer = lambda mlp: Y.attention_layer(H, max(H // 4, 1), D, CHUNK, Y.rotary(D, 1e6, factor=8.0, original=8192), mlp, softcap=30.0)
    return Y.pomisun(E, VOCAB, [layer(Y.dense_mlp(F)), layer(Y.moe_mlp(*EXPERTS[size]))] * 4)


def vifanex_config(size):
    from . import synth_stack as Y
    E, F, H, D = SIZES[size][:4]
    n, top, fe, fs = EXPERTS[size]
    dense, moe = Y.clamped_mlp(F, 7.0), Y.clamped_moe(n, top, fe, 7.0, shared=(fs, 7.0), groups=(8, 4), scale=2.5)
    att = lambda mlp: Y.normed_attention_layer(H, max(H // 4, 1), D, D, WINDOW, Y.banded_rotary(D, 1e6, factor=8.0, original=8192), mlp, v_mix=True)
    rec = lambda mlp: Y.channel_delta_layer(H, H, D, D, 4, mlp, 128, 128)
    return Y.vifanex(E, VOCAB, [att(dense), rec(moe), att(moe), rec(dense)] * 2, streams=4, softcap=30.0)


def kilurax_config(size):
    from . import synth_stack as Y
    E, F, H, D, _, _, MH, G = SIZES[size]
    moe = Y.moe_mlp(*EXPERTS[size])
    two = Y.parallel_mixer_layer((H, max(H // 4, 1), D, D), (MH, 64, 128, G, 4, G), (0.7, 0.4), Y.rotary(D, 1e6), moe)
    return Y.kilurax(E, VOCAB, [Y.delta_layer(H, H, D, D, 4, moe), two, Y.hgrn2_layer(H, D, D, moe), two] * 2, groups=4, taps=4,
                     pairs=(65536, 40503, 1))


def qwen3moe_shape(size):
    from . import gguf_writer as gw
    from . import synth
    E, F, H, D = SIZES[size][:4]
    n, top, fe, _ = EXPERTS[size]
    return synth.ModelShape("qwen3moe", 8, E, H, max(H // 4, 1), D, F, VOCAB, 500000.0, gw.GGML_Q4_K, n_expert=n, n_expert_used=top, n_ff_exp=fe,
                            name="qwen3moe-%s-mxfp4-8layers" % size)


def llama_shape(size):
    from . import gguf_writer as gw
    from . import synth
    E, F, H, D = SIZES[size][:4]
    return synth.ModelShape("llama", 8, E, H, max(H // 4, 1), D, F, VOCAB, 500000.0, gw.GGML_Q4_K, name="llama-%s-q4_k-8layers" % size)


def dibosun_work(cfg, rows, ctx, n_out):
    """Per category: (HBM bytes, bf16 flops, f32 flops) of a step of `rows` tokens that attend `ctx` keys each on
    average, its cached rows read once per block of tokens of one sequence (decode: once per row)."""
    E, T = cfg["width"], rows
    w = {k: [0.0, 0.0, 0.0] for k in ("norm", "qkv", "rope", "absorb", "attention", "o_proj", "scan", "down", "head")}

    def add(k, by, fl=0.0, f32=0.0):
        w[k][0] += by
        w[k][1] += fl
        w[k][2] += f32
    mat = lambda k, n, m, x, y: add(k, 2 * n * m + x * T * m + y * T * n, 2 * n * m * T)
    for layer in cfg["layers"]:
        m, F = layer["mixer"], layer["mlp"]["ff"]
        add("norm", T * E * (4 + 4 + 2))
        if layer["type"] == "latent_attention":
            H, D, V, Q, R = m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"]
            own = m.get("kv_from") is None
            n_in = Q + H + (R if own else 0)
            add("qkv", 2 * (n_in + F) * E + T * (2 * E + 4 * n_in + 2 * F), 2 * T * E * (n_in + F))
            add("rope", T * (4 * Q + 2 * Q + (4 * R + 2 * R if own else 0)))
            mat("absorb", H * D, Q, 2, 2)
            add("absorb", 2 * H * D * R + T * H * (2 * D + 2 * R), 2 * T * H * D * R)
            add("attention", ctx[1] * R * 2 + T * H * R * 4, 4 * T * H * ctx[0] * R)
            add("o_proj", 2 * H * V * R + T * H * (2 * R + 2 * V), 2 * T * H * V * R)
            mix = H * V
        else:
            mix, bc = m["heads"] * m["vdim"], 2 * m["groups"] * m["state"]
            n_in = 2 * mix + bc + m["heads"]
            add("qkv", 2 * (n_in + F) * E + T * (2 * E + 4 * n_in + 2 * F), 2 * T * E * (n_in + F))
            state = m["heads"] * m["state"] * m["vdim"]
            add("scan", 2 * 4 * state * ctx[2] + T * (4 * (mix + bc) + 4 * mix * 2 + 2 * mix), 0, 4 * T * state)
        add("down", 2 * E * (mix + F) + T * (2 * (mix + F) + 8 * E), 2 * T * E * (mix + F))
    add("head", 2 * cfg["vocab"] * E + n_out * (2 * E + 4 * cfg["vocab"]), 2 * n_out * E * cfg["vocab"])
    return w


def chosen_experts(n, top, rows):
    """Expected number of experts that some token of a step chooses (uniformly)."""
    return n * (1.0 - (1.0 - top / n) ** rows)


def pomisun_work(cfg, rows, ctx, n_out):
    E, T = cfg["width"], rows
    w = {}

    def add(k, by, fl=0.0):
        a = w.setdefault(k, [0.0, 0.0, 0.0])
        a[0] += by
        a[1] += fl
    for layer in cfg["layers"]:
        m, mlp = layer["mixer"], layer["mlp"]
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        add("norm", 2 * T * E * (4 + 4 + 2))
        add("qkv", 2 * (H + G) * D * E + T * (2 * E + 2 * H * D + 4 * G * D), 2 * T * E * (H + G) * D)
        add("attention", ctx[1] * 4 * G * D + T * H * D * 4, 4 * T * H * ctx[0] * D)
        add("o_proj", 2 * E * H * D + T * (2 * H * D + 8 * E), 2 * T * E * H * D)
        if mlp["kind"] == "dense":
            F = mlp["ff"]
            add("gate_up", 4 * F * E + T * (2 * E + 2 * F), 4 * T * E * F)
            add("down", 2 * E * F + T * (2 * F + 8 * E), 2 * T * E * F)
            continue
        n, top, F, S = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], mlp["shared"]["ff"]
        used = chosen_experts(n, top, T)
        add("shared", 2 * (n + 1 + 3 * S) * E + T * (2 * E + 4 * (n + 1) + 4 * S + 8 * E), 2 * T * E * (n + 1 + 3 * S))
        add("route", T * (4 * n + 8 * top))
        add("experts_in", 4 * used * F * E + T * 2 * E + T * top * 2 * F, 4 * T * top * E * F)
        add("experts_out", 2 * used * F * E + T * top * (2 * F + 4 * E), 2 * T * top * E * F)
    add("head", 2 * cfg["vocab"] * E + n_out * (2 * E + 4 * cfg["vocab"]), 2 * n_out * E * cfg["vocab"])
    return w


def vifanex_work(cfg, rows, ctx, n_out):
    E, T, s = cfg["width"], rows, cfg["streams"]
    w = {}

    def add(k, by, fl=0.0, f32=0.0):
        a = w.setdefault(k, [0.0, 0.0, 0.0])
        a[0] += by
        a[1] += fl
        a[2] += f32
    for layer in cfg["layers"]:
        m, mlp = layer["mixer"], layer["mlp"]
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        add("norm", 2 * T * E * (8 * s + 4 + 2))                 # every stream read and written, what is added, the activations
        if layer["type"] == "attention":
            n = (H + G) * D + G * V
            add("qkv", 2 * n * E + T * (2 * E + 4 * n), 2 * T * n * E)
            add("rope", T * (4 + 2) * n)
            add("attention", ctx[1] * 2 * G * (D + V) + T * H * 2 * (D + V), 2 * T * H * ctx[0] * (D + V))
        else:
            n, ra, rg = 2 * G * D + H * V + H, m["decay_rank"], m["gate_rank"]
            add("qkv", 2 * (n + ra + rg) * E + T * (2 * E + 4 * n + 2 * (ra + rg)), 2 * T * (n + ra + rg) * E)
            add("low_rank", 2 * H * (D * ra + V * rg) + T * (2 * (ra + rg) + 4 * H * (D + V)), 2 * T * H * (D * ra + V * rg))
            add("scan", 8 * H * D * V * ctx[2] + T * (4 * n + 4 * H * (D + V) + 2 * H * V), 0, 6 * T * H * D * V)
        add("o_proj", 2 * E * H * V + T * (2 * H * V + 4 * E), 2 * T * E * H * V)
        if mlp["kind"] == "dense":
            F = mlp["ff"]
            add("gate_up", 4 * F * E + T * (2 * E + 2 * F), 4 * T * E * F)
            add("down", 2 * E * F + T * (2 * F + 4 * E), 2 * T * E * F)
            continue
        n, top, F, S = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], mlp["shared"]["ff"]
        used = chosen_experts(n, top, T)
        add("shared", 2 * (n + 3 * S) * E + T * (2 * E + 4 * n + 4 * S + 4 * E), 2 * T * E * (n + 3 * S))
        add("route", T * (4 * n + 8 * top))
        add("experts_in", 4 * used * F * E + T * 2 * E + T * top * 2 * F, 4 * T * top * E * F)
        add("experts_out", 2 * used * F * E + T * top * (2 * F + 4 * E), 2 * T * top * E * F)
    add("head", 2 * cfg["vocab"] * E + n_out * (2 * E + 4 * cfg["vocab"]), 2 * n_out * E * cfg["vocab"])
    return w


def kilurax_work(cfg, rows, ctx, n_out):
    E, T = cfg["width"], rows
    w = {}

    def add(k, by, fl=0.0, f32=0.0):
        a = w.setdefault(k, [0.0, 0.0, 0.0])
        a[0] += by
        a[1] += fl
        a[2] += f32
    for layer in cfg["layers"]:
        m, mlp = layer["mixer"], layer["mlp"]
        add("norm", 2 * T * E * (8 + 4 + 2))                     # the stream read and written, what is added, the activations
        if layer["type"] == "parallel":
            a, s = m["left"], m["right"]
            H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            n_a, mix, bc = (H + G) * D + G * V, s["heads"] * s["vdim"], 2 * s["groups"] * s["state"]
            n_s, state = 2 * mix + bc + s["heads"], s["heads"] * s["state"] * s["vdim"]
            add("qkv", 2 * (n_a + n_s) * E + T * (2 * E + 2 * n_a + 4 * n_s), 2 * T * (n_a + n_s) * E)
            add("attention", ctx[1] * 2 * G * (D + V) + T * H * 2 * (D + V), 2 * T * H * ctx[0] * (D + V))
            add("scan", 8 * state * ctx[2] + T * (4 * (mix + bc) + 8 * mix + 2 * mix), 0, 4 * T * state)
            n_o = H * V + mix
        else:
            H, D, V = m["heads"], m["dim"], m["vdim"]
            G, per = m.get("kv_heads", H), 6 if layer["type"] == "delta" else 4
            n = 2 * G * D + H * V + (2 * H + H * V if layer["type"] == "delta" else 0)
            add("qkv", 2 * n * E + T * (2 * E + 4 * n), 2 * T * n * E)
            add("scan", 8 * H * D * V * ctx[2] + T * (4 * n + 2 * H * V), 0, per * T * H * D * V)
            n_o = H * V
        add("o_proj", 2 * E * n_o + T * (2 * n_o + 4 * E), 2 * T * E * n_o)
        n, top, F, S = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], mlp["shared"]["ff"]
        used = chosen_experts(n, top, T)
        add("shared", 2 * (n + 3 * S) * E + T * (2 * E + 4 * n + 4 * S + 4 * E), 2 * T * E * (n + 3 * S))
        add("route", T * (4 * n + 8 * top))
        add("experts_in", 4 * used * F * E + T * 2 * E + T * top * 2 * F, 4 * T * top * E * F)
        add("experts_out", 2 * used * F * E + T * top * (2 * F + 4 * E), 2 * T * top * E * F)
    add("embed", T * E * 8)
    add("head", 2 * cfg["vocab"] * E + n_out * (2 * E + 4 * cfg["vocab"]), 2 * n_out * E * cfg["vocab"])
    return w


def qwen3moe_work(s, rows, ctx, n_out):
    from . import gguf_writer as gw
    w = llama_work(s, rows, ctx, n_out)
    el, by = gw.BLOCK_GEOMETRY[s.expert_type]
    E, F, top = s.n_embd, s.n_ff_exp, s.n_expert_used
    used = chosen_experts(s.n_expert, top, rows)
    # one category: router, routing, gate/up and down of the experts
    w["gate_up"] = (s.n_layer * (4 * s.n_expert * E + 3 * used * E * F * by / el + rows * (4 * E + top * (4 * F + 4 * E))),
                    s.n_layer * 2 * rows * E * (s.n_expert + 3 * top * F), 0.0)
    return w


def llama_work(s, rows, ctx, n_out):
    from . import gguf_writer as gw
    el, by = gw.BLOCK_GEOMETRY[s.matrix_type]
    E, T, L = s.n_embd, rows, s.n_layer
    QD, KD, F = s.n_head * s.head_dim, s.n_head_kv * s.head_dim, s.n_ff
    mat = lambda n, m: (L * (n * m * by / el + T * 4 * (n + m)), L * 2 * n * m * T, 0.0)
    return {"norm": (2 * L * T * E * 12, 0.0, 0.0), "qkv": mat(QD + 2 * KD, E), "o_proj": mat(E, QD), "gate_up": mat(2 * F, E),
            "down": mat(E, F), "attention": (L * (ctx[1] * 4 * KD + T * QD * 8), L * 4 * T * QD * ctx[0], 0.0),
            "head": (s.n_vocab * E * by / el + n_out * 4 * (E + s.n_vocab), 2 * n_out * E * s.n_vocab, 0.0)}


def roofline(work):
    return max(work[0] / HBM, work[1] / BF16, work[2] / F32)


MOE = ("shared", "route", "experts_in", "experts_out")       # what a mixture of experts consists of, also reported as one


def categories(prof, n_steps, work):
    out = {}
    if prof.get("route", (0, 0))[1]:
        parts = [k for k in MOE if k in prof]
        prof = dict(prof, moe=(sum(prof[k][0] for k in parts), sum(prof[k][1] for k in parts)))
        work = dict(work, moe=[sum(work[k][i] for k in parts) for i in range(3)])
    for k, (ms, n) in sorted(prof.items(), key=lambda kv: -kv[1][0]):
        if n:
            out[k] = {"us": round(ms / n_steps * 1e3, 1), "launches": n // n_steps}
            if k in work:
                out[k]["of_roofline"] = round(roofline(work[k]) / (ms / n_steps * 1e-3), 3)
    return out


def measure(path, E, vocab, work_of, keys_of, n_batch, prefill_sizes, steps):
    """keys_of: positions -> the number of keys a token there attends."""
    import torch

    n_ctx = N_SEQ_MAX * (CONTEXT + 128) + 8192
    eng = E.Engine(path, E.EngineConfig(n_ctx=n_ctx, n_seq_max=N_SEQ_MAX + 1, n_batch=n_batch, n_ubatch=n_batch))
    torch.cuda.empty_cache()
    rng = np.random.default_rng(5)
    out = {"prefill": {}, "decode": {}}
    step_out = E.StepOutput(N_SEQ_MAX + 1)
    greedy = E.SamplingParamsV2.greedy()
    draw = lambda n: rng.integers(0, vocab, n).astype(np.int32)

    def timed(rows, repeat, after):
        """Median seconds of a step run `repeat` times, then its kernel categories over two more runs."""
        secs = []
        for i in range(repeat + 4):
            eng.profile(2 if i >= repeat + 2 else 0)
            if i == repeat + 2:
                eng.profile_read(reset=True)
            r = rows(i)
            t0 = time.perf_counter()
            eng.step(r, step_out)
            if 2 <= i < repeat + 2:
                secs.append(time.perf_counter() - t0)
            after(i)
        prof = eng.profile_read(reset=True)
        eng.profile(0)
        return float(np.median(secs)), prof

    for n in prefill_sizes:
        toks = draw(n)
        sec, prof = timed(lambda i: [E.StepRow(0, 0, toks, 0, sample=True, sampling=greedy)], 8, lambda i: (eng.seq_rm(0), eng.request_free(0)))
        keys = float(np.mean(keys_of(np.arange(n))))
        out["prefill"][n] = {"ms": round(sec * 1e3, 3), "tok_s": round(n / sec, 1),
                             "kernels": categories(prof, 2, work_of(n, (keys, n, 1), 1))}
        print("[bench] prefill", n, json.dumps(out["prefill"][n]), file=sys.stderr, flush=True)
    for s in range(N_SEQ_MAX):
        toks = draw(CONTEXT)
        for at in range(0, CONTEXT, n_batch):
            eng.step([E.StepRow(s, s, toks[at:at + n_batch], at, sample=True, sampling=greedy)], step_out)
    pos = [CONTEXT] * N_SEQ_MAX
    for n in (1, 16, 64):
        def advance(i):
            for s in range(n):
                pos[s] += 1
        at = pos[0]
        sec, prof = timed(lambda i: [E.StepRow.decode(s, s, int(7 * s + i) % vocab, pos[s], greedy) for s in range(n)], steps, advance)
        keys = float(np.mean(keys_of(at + np.arange(steps))))
        out["decode"][n] = {"ms": round(sec * 1e3, 3), "tok_s": round(n / sec, 1),
                            "kernels": categories(prof, 2, work_of(n, (keys, keys * n, n), n))}
        print("[bench] decode", n, json.dumps(out["decode"][n]), file=sys.stderr, flush=True)
    eng.close()
    return out


def main(args) -> int:
    import torch

    from . import engine as E
    from . import synth
    from . import synth_stack as Y

    if not torch.cuda.is_available():
        print("this benchmark needs an MI355X: no HIP device is visible", file=sys.stderr)
        return 2
    causal, windowed, chunked = lambda p: p + 1, lambda p: np.minimum(p + 1, WINDOW), lambda p: p % CHUNK + 1
    stacks = {"dibosun": (dibosun_config, dibosun_work, windowed), "pomisun": (pomisun_config, pomisun_work, chunked), "vifanex": (vifanex_config, vifanex_work, windowed),
              "kilurax": (kilurax_config, kilurax_work, causal)}
    ggufs = {"llama": (llama_shape, llama_work), "qwen3moe": (qwen3moe_shape, qwen3moe_work)}
    closest = {"dibosun": ["llama"], "pomisun": ["llama", "qwen3moe"], "vifanex": ["pomisun", "dibosun"], "kilurax": ["vifanex", "pomisun", "dibosun"]}[args.model]
    steps = min(args.steps, 16)
    result = {"metric": "prefill and decode throughput, %s beside other models (GGUF ones in Q4_K, MXFP4 experts) of equal width, feed-forward and depth" % args.model.capitalize(),
              "data": "synthetic", "context": CONTEXT, "vocab": VOCAB, "layers": 8, "sizes": {}}
    for size in args.stack_sizes.split(","):
        entry = {}
        for name in [args.model] + ([] if args.no_closest_model else closest):
            print("[bench]", name, size, file=sys.stderr, flush=True)
            if name in stacks:
                config_of, work, keys = stacks[name]
                cfg = config_of(size)
                path = Path(args.model_dir) / ("retro-bench-%s-%s" % (name, size))
                if not (path / "done").exists():
                    Y.write_random_checkpoint(path, cfg, args.seed)
                    (path / "done").write_text("")
                work_of = lambda *a: work(cfg, *a)
            else:
                shape_of, work = ggufs[name]
                shape, keys = shape_of(size), causal
                path = Path(args.model_dir) / ("retro-bench-%s.gguf" % shape.name)
                if not path.exists():
                    synth.write_model(path.with_suffix(".tmp"), shape, seed=args.seed, device="cuda")
                    os.replace(path.with_suffix(".tmp"), path)
                work_of = lambda *a: work(shape, *a)
            entry[name] = measure(path, E, VOCAB, work_of, keys, 4096, (512, 4096), steps)
        result["sizes"][size] = entry
    print(json.dumps(result), flush=True)
    return 0
