"""What the GPU tests of layer-stack models share: a random checkpoint with its plain statement, and comparisons."""
import numpy as np
import pytest

import plain_kilurax
import plain_layers
import plain_pomisun
import plain_vifanex
from retrograd_amd import engine as E
from retrograd_amd import synth_stack as Y

PLAIN = {"Dibosun": plain_layers, "Pomisun": plain_pomisun, "Vifanex": plain_vifanex, "Kilurax": plain_kilurax}

LIMIT = {E.KV_F32: 3e-5, E.KV_F16: 0.035}
KINDS = [pytest.param(E.KV_F32, id="f32"), pytest.param(E.KV_F16, id="bf16")]


class Model:
    def __init__(self, folder, cfg, edit=None):
        self.cfg = cfg
        self.tensors = Y.random_tensors(self.cfg, 11)
        if edit:
            edit(self.cfg, self.tensors)
            self.tensors = {k: Y.from_bf16(Y.to_bf16(v)) for k, v in self.tensors.items()}
        self.folder = Y.write_checkpoint(folder, self.cfg, self.tensors)
        self.seen = {}

    def plain(self, tokens):
        key = tuple(int(t) for t in tokens)
        if key not in self.seen:
            self.seen[key] = PLAIN[self.cfg["architecture"]].run_stack(self.cfg, self.tensors, tokens)
        return self.seen[key]

    def tokens(self, n, seed=0):
        return np.random.default_rng(seed + 100).integers(0, self.cfg["vocab"], n)

    def engine(self, kv, n_ctx=640, slots=4, n_batch=256):
        print("engine", self.folder.name, "kv", kv, flush=True)
        return E.Engine(self.folder, E.EngineConfig(n_ctx=n_ctx, n_seq_max=slots, n_batch=n_batch, n_ubatch=n_batch, kv_dtype=kv))


def close(got, want, kv, what=""):
    """Root mean square over the vocabulary, relative to the logits' own."""
    got, want = np.atleast_2d(got).astype(np.float64), np.atleast_2d(want)
    d = got - want
    err = np.sqrt((d * d).mean(1)) / np.sqrt((want * want).mean())
    assert np.isfinite(got).all() and err.max() <= LIMIT[kv], (what, int(err.argmax()), float(err.max()))


def feed(eng, slot, tokens, sizes, at=0):
    """The tokens in portions (the last size repeats); all logits."""
    out, i = [], 0
    while at < len(tokens):
        n = min(sizes[min(i, len(sizes) - 1)], len(tokens) - at)
        out.append(eng.step_logits([(slot, tokens[at:at + n], at)], [(0, k) for k in range(n)]))
        at += n
        i += 1
    return np.concatenate(out)


def plain_greedy(m, prompt, n):
    """Greedy continuation, and the smallest lead of a chosen token over the next in units of the logits' spread."""
    toks, lead = list(prompt), np.inf
    for _ in range(n):
        row = PLAIN[m.cfg["architecture"]].run_stack(m.cfg, m.tensors, toks)[-1]
        a, b = np.sort(row)[-2:]
        lead = min(lead, (b - a) / row.std())
        toks.append(int(row.argmax()))
    return toks[len(prompt):], lead
