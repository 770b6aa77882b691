"""Prefill and decode of layer-stack models (Dibosun) at sizes that resemble a real model's layers, beside the closest
GGUF model of the same width, feed-forward width and depth: what `bench.py --model dibosun` runs. Weights are random
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
VOCAB, WINDOW = 32000, 1024


def dibosun_config(size):
    from . import synth_stack as Y
    E, F, H, D, QR, R, MH, G = SIZES[size]
    lat = lambda kv_from=None: Y.latent_layer(H, D, D, QR, R, WINDOW, F, kv_from=kv_from)
    mam = lambda: Y.mamba2_layer(MH, 64, 128, G, 4, G, F)
    return Y.dibosun(E, VOCAB, [lat(), mam(), lat(0), mam(), lat(), mam(), lat(4), mam()])


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


def categories(prof, n_steps, work):
    out = {}
    for k, (ms, n) in sorted(prof.items(), key=lambda kv: -kv[1][0]):
        if n:
            out[k] = {"us": round(ms / n_steps * 1e3, 1), "launches": n // n_steps}
            if k in work:
                out[k]["of_roofline"] = round(roofline(work[k]) / (ms / n_steps * 1e-3), 3)
    return out


def measure(path, E, vocab, work_of, window, n_batch, prefill_sizes, steps):
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
        keys = float(np.mean(np.minimum(np.arange(n) + 1, window)))
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
        keys = float(min(at + steps / 2, window))
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
    sizes = args.stack_sizes.split(",")
    steps = min(args.steps, 16)
    result = {"metric": "prefill and decode throughput, Dibosun beside Llama (Q4_K) of equal width, feed-forward and depth",
              "data": "synthetic", "context": CONTEXT, "window": WINDOW, "vocab": VOCAB, "layers": 8, "sizes": {}}
    for size in sizes:
        cfg = dibosun_config(size)
        folder = Path(args.model_dir) / ("retro-bench-dibosun-%s" % size)
        if not (folder / "done").exists():
            Y.write_random_checkpoint(folder, cfg, args.seed)
            (folder / "done").write_text("")
        print("[bench] dibosun", size, file=sys.stderr, flush=True)
        entry = {"dibosun": measure(folder, E, VOCAB, lambda *a: dibosun_work(cfg, *a), WINDOW, 4096, (512, 4096), steps)}
        if not args.no_closest_model:
            shape = llama_shape(size)
            path = Path(args.model_dir) / ("retro-bench-%s.gguf" % shape.name)
            if not path.exists():
                synth.write_model(path.with_suffix(".tmp"), shape, seed=args.seed, device="cuda")
                os.replace(path.with_suffix(".tmp"), path)
            print("[bench] llama", size, file=sys.stderr, flush=True)
            entry["llama"] = measure(path, E, VOCAB, lambda *a: llama_work(shape, *a), 1 << 30, 4096, (512, 4096), steps)
        result["sizes"][size] = entry
    print(json.dumps(result), flush=True)
    return 0
