"""The Vifanex design through the engine against the plain statements in plain_vifanex.py: the gated delta rule with a decay
per key channel, windowed attention with normed queries and keys and mixed values, several residual streams, clamped gated
feed-forwards and routing over groups of experts. Every mechanism alone and together, prompts against decoding and portions,
batches, reused pages and slots."""
import io
import json

import numpy as np
import pytest

import plain_vifanex as P
from plain_layers import rms_norm
from retrograd_amd import engine as E
from retrograd_amd import scheduler as S
from retrograd_amd import synth_stack as Y
from stack_helpers import KINDS, LIMIT, Model, close, feed, plain_greedy

pytestmark = pytest.mark.gpu

STRETCHED = Y.banded_rotary(12, 500.0, factor=6.0, original=50, high=5.0, low=1.5)


def attention(heads=6, kv_heads=2, dim=20, vdim=28, window=45, rot=STRETCHED, mlp=None, **kw):
    return Y.normed_attention_layer(heads, kv_heads, dim, vdim, window, rot, mlp, **kw)


def delta(heads=4, kv_heads=2, dim=20, vdim=24, conv=3, mlp=None, decay_rank=9, gate_rank=14):
    return Y.channel_delta_layer(heads, kv_heads, dim, vdim, conv, mlp, decay_rank, gate_rank)


def model(*layers, width=72, vocab=40, **kw):
    return Y.vifanex(width, vocab, list(layers), **kw)


CONFIGS = {
    # each mechanism alone
    "attention": model(attention(rot=Y.banded_rotary(20)), streams=1),
    "attention-unbounded": model(attention(window=None)),
    "rotary-partial": model(attention(rot=Y.banded_rotary(8, 300.0))),
    "rotary-none": model(attention(rot=None)),
    "rotary-stretched": model(attention()),
    "values-narrow": model(attention(dim=66, vdim=9)),
    "values-wide": model(attention(dim=7, vdim=50, rot=Y.banded_rotary(6))),
    "values-mixed": model(attention(v_mix=True), attention(window=20, kv_heads=1, vdim=56, v_mix=False), attention(heads=2, kv_heads=1, vdim=56, v_mix=True), attention(v_mix=True)),
    "delta": model(delta()),
    "delta-shared-keys": model(delta(heads=6, kv_heads=1)),
    "delta-own-keys": model(delta(heads=3, kv_heads=3, conv=4)),
    "delta-no-convolution": model(delta(conv=1)),
    "delta-long-taps": model(delta(conv=6)),
    "delta-two-taps": model(delta(conv=2, decay_rank=40, gate_rank=3)),
    "streams-one": model(delta(mlp=Y.clamped_mlp(30)), streams=1),
    "streams-four": model(attention(mlp=Y.clamped_mlp(30)), delta(), streams=4),
    "streams-many": model(delta(mlp=Y.clamped_mlp(30)), attention(), streams=7),
    "dense": model(attention(mlp=Y.clamped_mlp(50, 0.6))),
    "dense-high-limit": model(attention(mlp=Y.clamped_mlp(50, 100.0))),
    "experts": model(attention(mlp=Y.clamped_moe(6, 2, 40))),
    "experts-shared": model(attention(mlp=Y.clamped_moe(6, 3, 20, 0.7, shared=(50, 1.9), scale=2.5))),
    "experts-groups": model(attention(mlp=Y.clamped_moe(12, 3, 20, groups=(4, 2), scale=1.7))),
    "experts-groups-all": model(attention(mlp=Y.clamped_moe(6, 6, 12, groups=(3, 3), shared=(8, 1.0)))),
    "experts-group-each": model(attention(mlp=Y.clamped_moe(5, 2, 12, groups=(5, 2)))),
    "experts-many": model(attention(mlp=Y.clamped_moe(300, 5, 9, shared=(33, 1.0), groups=(6, 2)))),
    "experts-one": model(attention(mlp=Y.clamped_moe(1, 1, 30))),
    "uncapped": dict(model(delta()), logit_softcap=None),
    # together, every layer of other sizes; the width is no multiple of a tile
    "all": model(
        delta(mlp=Y.clamped_moe(8, 2, 33, 0.8, shared=(41, 2.5), groups=(4, 2), scale=1.3)),
        attention(mlp=Y.clamped_mlp(90, 1.1), v_mix=True),
        attention(heads=3, kv_heads=3, dim=40, vdim=17, window=33, rot=Y.banded_rotary(40, 300.0)),
        delta(heads=3, kv_heads=3, dim=37, vdim=11, conv=4, mlp=Y.clamped_mlp(20), decay_rank=50, gate_rank=7),
        attention(heads=8, kv_heads=1, dim=18, vdim=56, window=70, v_mix=True, mlp=Y.clamped_moe(9, 3, 20), scale=0.5),
        delta(heads=10, kv_heads=2, dim=70, vdim=34, conv=2),
        attention(heads=4, kv_heads=4, dim=66, vdim=14, window=9, rot=Y.banded_rotary(22, 90.0), v_mix=True),
        width=107, vocab=50, streams=3, eps=1e-4, softcap=12.0, embedding_scale=3.0),
    # sizes of one
    "ones": model(
        attention(heads=1, kv_heads=1, dim=1, vdim=1, window=1, rot=Y.banded_rotary(0), mlp=Y.clamped_moe(1, 1, 1, shared=(1, 1.0)), scale=1.5, v_mix=True),
        delta(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, mlp=Y.clamped_mlp(1), decay_rank=1, gate_rank=1),
        attention(heads=2, kv_heads=1, dim=2, vdim=1, window=2, rot=Y.banded_rotary(2, 7.0), v_mix=True), width=9, vocab=5),
    # sizes of a real model's heads and experts
    "wide": model(
        attention(heads=16, kv_heads=4, dim=128, vdim=128, window=100, rot=Y.banded_rotary(128, 1e5, factor=4.0, original=64), mlp=Y.clamped_mlp(1536), v_mix=True),
        delta(heads=8, kv_heads=4, dim=128, vdim=128, conv=4, mlp=Y.clamped_moe(16, 4, 512, shared=(544, 3.0), groups=(4, 2), scale=2.0), decay_rank=128, gate_rank=128),
        attention(heads=40, kv_heads=4, dim=64, vdim=128, window=150, rot=Y.banded_rotary(32), v_mix=True, mlp=Y.clamped_moe(12, 3, 160)),
        delta(heads=6, kv_heads=6, dim=96, vdim=200, conv=4, decay_rank=64, gate_rank=100), width=512, vocab=150, streams=4, embedding_scale=2.0),
}
BIG = ["all", "ones", "wide"]


def decide_routing(cfg, tensors):
    """Routers that follow the token: the kept groups and the chosen experts stand clear of the others, so that rounding
    chooses no other expert (a test of rounding must not rest on a close call)."""
    rng = np.random.default_rng(1)
    tensors["embed"] = 5.0 * tensors["embed"]
    for i, layer in enumerate(cfg["layers"]):
        if not layer.get("mlp") or layer["mlp"]["kind"] != "moe":
            continue
        r = layer["mlp"]["router"]
        g = r.get("groups", {"count": 1, "keep": 1})
        size = r["experts"] // g["count"]
        h = rms_norm(tensors["embed"], tensors["l%d.norm2" % i], cfg["norm"]["eps"])
        z = rng.uniform(-1.0, 1.0, (cfg["vocab"], r["experts"]))
        for row in z:
            kept = rng.permutation(g["count"])[:g["keep"]]
            inside = np.concatenate([rng.permutation(np.arange(k * size, (k + 1) * size)) for k in kept])
            firsts = inside[::size]                                  # one expert of every kept group, then any others
            others = rng.permutation(np.setdiff1d(inside, firsts))
            row[np.concatenate([firsts, others])[:max(r["top"], len(firsts))]] += 7.0
            if len(firsts) > r["top"]:                               # kept groups beyond the chosen experts: their best comes behind
                row[firsts[r["top"]:]] -= 3.0
        tensors["l%d.mlp.router" % i] = np.linalg.lstsq(h, z, rcond=None)[0].T.astype(np.float32)


class Vifanex(Model):
    """Its plain statement also makes sure that the routing is decided."""
    def plain(self, tokens):
        key = tuple(int(t) for t in tokens)
        if key not in self.seen:
            leads = []
            self.seen[key] = P.run_stack(self.cfg, self.tensors, tokens, leads=leads)
            assert all(lead.min() > 0.05 for lead in leads), [float(lead.min()) for lead in leads]
        return self.seen[key]


def steer(cfg, tensors):
    """Routing decided by the token at any depth: every sublayer reads a first stream that only ever holds the embedding."""
    decide_routing(cfg, tensors)
    if not any((layer.get("mlp") or {}).get("kind") == "moe" for layer in cfg["layers"]):
        return
    for name in list(tensors):
        n = cfg["streams"]
        if ".hc" not in name:
            continue
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "mix":
            tensors[name][:, 0] = 0.0
            tensors[name][0, 0] = 1.0
        elif leaf == "out":
            tensors[name][0] = 0.1 if n > 1 else 0.3
        elif ".hc2." in name:
            tensors[name][0] = 1.0
            tensors[name][1:] *= 0.15


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Vifanex(tmp_path_factory.mktemp("vifanex") / name, CONFIGS[name], steer)
        return made[name]
    return get


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts_and_every_layer(models, name, kv):
    m = models(name)
    with m.engine(kv) as eng:
        eng.keep_residual(True)
        for n in (1, 2, 3, 17, 150):
            toks = m.tokens(n, n)
            got = eng.step_logits([(0, toks, 0)], [(0, k) for k in range(n)])
            close(got, m.plain(toks), kv, n)
            keep = []
            P.run_stack(m.cfg, m.tensors, toks, keep=keep)
            res = eng.residual(len(keep), m.cfg["width"])
            for layer, (a, b) in enumerate(zip(res, keep)):
                close(a, b, kv, (n, "layer", layer))
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", BIG + ["delta", "delta-long-taps", "values-mixed", "values-narrow", "experts-groups", "streams-many"])
def test_token_by_token_is_the_prompt(models, name, kv):
    m = models(name)
    toks = m.tokens(130)
    with m.engine(kv) as eng:
        close(feed(eng, 1, toks, [1]), m.plain(toks), kv)
        eng.seq_rm(1)
        close(feed(eng, 2, toks, [77, 1]), m.plain(toks), kv)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", BIG + ["delta-no-convolution"])
def test_portions_of_any_size(models, name, kv):
    m = models(name)
    toks = m.tokens(150)
    with m.engine(kv) as eng:
        for sizes in ([2], [3], [7, 2, 31, 5], [16], [32], [33, 31, 2], [64, 65], [128, 2], [149, 1]):
            close(feed(eng, 0, toks, sizes), m.plain(toks), kv, sizes)
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", ["all", "wide"])
def test_mixed_batches_pages_and_slots_used_again(models, name, kv):
    """Requests of unequal lengths come and go in four slots of a pool that only holds what is live: prompt portions
    beside single tokens, every logit against the request alone."""
    m = models(name)
    rng = np.random.default_rng(3)
    todo = [(i, m.tokens(int(n), i)) for i, n in enumerate((150, 40, 97, 1, 2, 131, 64, 33, 150, 75, 20, 5))]
    live, free, got = {}, [0, 1, 2, 3], {i: [] for i, _ in todo}
    with m.engine(kv, n_ctx=640, slots=4) as eng:
        while todo or live:
            while todo and free:
                i, toks = todo.pop(0)
                live[i] = [free.pop(), toks, 0]
            rows, want, names = [], [], []
            for i, (slot, toks, at) in live.items():
                if len(live) > 1 and rng.random() < 0.15 and rows:
                    continue                                  # left out of this step
                n = min(len(toks) - at, 1 if at and rng.random() < 0.5 else int(rng.integers(1, 80)))
                want += [(len(rows), k) for k in range(n)]
                names += [i] * n
                rows.append((slot, toks[at:at + n], at))
                live[i][2] += n
            for i, row in zip(names, eng.step_logits(rows, want)):
                got[i].append(row)
            for i in [i for i, v in live.items() if v[2] == len(v[1])]:
                eng.seq_rm(live[i][0])
                free.append(live[i][0])
                close(np.array(got[i]), m.plain(live[i][1]), kv, i)
                del live[i]


@pytest.mark.parametrize("kv", KINDS)
def test_several_rows_of_one_slot_in_one_step(models, kv):
    m = models("all")
    toks, other = m.tokens(90), m.tokens(30, 5)
    with m.engine(kv) as eng:
        rows = [(2, toks[:2], 0), (0, other[:11], 0), (2, toks[2:40], 2), (2, toks[40:], 40), (0, other[11:], 11)]
        want = [(r, k) for r, (_, t, _) in enumerate(rows) for k in range(len(t))]
        got = eng.step_logits(rows, want)
        pick = lambda slot: np.array([g for g, (r, _) in zip(got, want) if rows[r][0] == slot])
        close(pick(2), m.plain(toks), kv)
        close(pick(0), m.plain(other), kv)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", ["all", "wide"])
def test_many_decoding_sequences(models, name, kv):
    """Decode-only batches of every size class of the product kernels, each sequence at another length."""
    m = models(name)
    n_seq = 70
    prompts = [m.tokens(3 + (7 * i) % 60, i % 9) for i in range(n_seq)]
    with m.engine(kv, n_ctx=n_seq * 96, slots=n_seq, n_batch=4096) as eng:
        eng.step_logits([(i, p[:-3], 0) for i, p in enumerate(prompts) if len(p) > 3], [])
        for count, k in ((70, -3), (33, -2), (9, -1)):
            rows = [(i, [prompts[i][k]], len(prompts[i]) + k) for i in range(count)]
            got = eng.step_logits(rows, [(r, 0) for r in range(count)])
            for i in list(range(0, count, 5)) + [count - 1]:
                close(got[i], m.plain(prompts[i])[len(prompts[i]) + k], kv, (count, i))


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("dim, vdim", [(6, 30), (96, 20), (50, 100), (120, 40), (160, 128), (200, 66), (100, 250), (256, 256), (270, 90), (40, 300)])
def test_key_and_value_widths(tmp_path, dim, vdim, kv):
    """Pairs of widths the attention kernels are compiled for, rounded up to and beyond them, with few, some and many query
    heads per key head: whole prompts, decoding one sequence (whose keys are shared out) and many."""
    for heads, kv_heads in ((5, 5), (40, 2), (20, 1)):
        m = Vifanex(tmp_path / ("d%dh%dg%d" % (dim, heads, kv_heads)), model(
            attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=150, rot=Y.banded_rotary(dim // 4 * 2), scale=2 * dim ** -0.5), width=48, vocab=60))
        toks = m.tokens(230, heads)
        want = m.plain(toks)
        with m.engine(kv, n_ctx=256 * 12, slots=12) as eng:
            close(feed(eng, 0, toks, [227, 1]), want, kv, (heads, kv_heads, "one"))
            for s in range(1, 12):
                eng.step_logits([(s, toks[:20 * s], 0)], [])
            got = eng.step_logits([(s, [toks[20 * s]], 20 * s) for s in range(1, 12)], [(s, 0) for s in range(11)])
            close(got, want[[20 * s for s in range(1, 12)]], kv, (heads, kv_heads, "many"))


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("heads, kv_heads, dim, vdim", [(2, 1, 5, 3), (3, 3, 16, 32), (2, 2, 40, 70), (4, 2, 64, 130), (2, 1, 90, 33), (2, 2, 128, 260), (2, 1, 140, 64), (1, 1, 300, 50), (2, 2, 33, 600)])
def test_state_sizes(tmp_path, heads, kv_heads, dim, vdim, kv):
    """Every shape of the recurrence's kernels: heads too wide for the chunks or for one block of columns among them."""
    m = Vifanex(tmp_path / "state", model(delta(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=4), width=60, vocab=50))
    toks = m.tokens(200, dim)
    want = m.plain(toks)
    with m.engine(kv) as eng:
        for sizes in ([200], [1], [70, 3, 1, 32, 31]):
            close(feed(eng, 0, toks, sizes), want, kv, sizes)
            eng.seq_rm(0)


def decays(a_log, bias):
    def edit(cfg, tensors):
        for name in tensors:
            if name.endswith("A_log"):
                tensors[name] = np.linspace(*a_log, tensors[name].size).astype(np.float32)
            elif name.endswith("dt_bias"):
                tensors[name] = np.linspace(*bias, tensors[name].size).astype(np.float32)[np.random.default_rng(0).permutation(tensors[name].size)]
    return edit


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name, a_log, bias", [("none", (-12.0, -9.0), (-6.0, -4.0)), ("all", (2.0, 4.0), (-1.0, 6.0)), ("both", (-5.0, 3.0), (-8.0, 5.0))])
def test_weak_and_strong_decays(tmp_path, name, a_log, bias, kv):
    """Channels that forget nothing over the whole prompt beside channels that forget everything at every token."""
    m = Vifanex(tmp_path / name, model(delta(heads=4, kv_heads=2, dim=48, vdim=32), delta(heads=2, kv_heads=2, dim=24, vdim=40)), decays(a_log, bias))
    toks = m.tokens(300, 1)
    want = m.plain(toks)
    with m.engine(kv, n_batch=320) as eng:
        for sizes in ([300], [1], [100, 33, 2]):
            close(feed(eng, 0, toks, sizes), want, kv, (name, sizes))
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
def test_a_write_is_read_far_away(tmp_path, kv):
    """One token's key stands alone: nothing else is written to its channel and nothing decays there, so what it wrote decides
    read-outs hundreds of tokens later, across chunks, steps and decoding; without it the output is another."""
    def edit(cfg, tensors):
        decays((-9.0, -8.0), (-6.0, -5.0))(cfg, tensors)
        for n in ("q", "k", "v"):
            tensors["l0.mix.%s.conv" % n] = np.tile([0.0, 0.0, 1.0], (len(tensors["l0.mix.%s.conv" % n]), 1)).astype(np.float32)
        E_ = np.zeros((cfg["vocab"], cfg["width"]))
        E_[np.arange(cfg["vocab"]), np.arange(cfg["vocab"])] = 1.0                 # a column per token
        tensors["embed"] = E_.astype(np.float32)
        D = cfg["layers"][0]["mixer"]["dim"]
        k, q = np.zeros((D, cfg["width"])), np.zeros((D, cfg["width"]))
        k[1:, :cfg["vocab"]] = np.random.default_rng(2).uniform(0.5, 1.0, (D - 1, cfg["vocab"]))
        k[:, 7] = 0.0
        k[0, 7] = 1.0                                                               # token 7 writes to channel 0
        k[0, 8:cfg["vocab"]] = -12.0                                                # ... which SiLU closes for every other
        k[0, :7] = -12.0
        q[0] = 1.0
        q[1:] = -12.0
        tensors["l0.mix.k"], tensors["l0.mix.q"] = (4.0 * k).astype(np.float32), (4.0 * q).astype(np.float32)
    m = Vifanex(tmp_path / "far", model(delta(heads=1, kv_heads=1, dim=16, vdim=24), width=60, vocab=50), edit)
    for place in (0, 31, 63, 64, 100):
        toks = m.tokens(420, place)
        toks[toks == 7] = 8
        without = P.run_stack(m.cfg, m.tensors, toks)[-8:]
        toks[place] = 7
        want = m.plain(toks)
        off = without - want[-8:]
        assert np.sqrt((off * off).mean(1)).min() > 2 * LIMIT[kv] * np.sqrt((want * want).mean())
        with m.engine(kv, n_ctx=2048, n_batch=512) as eng:
            close(feed(eng, 0, toks, [420]), want, kv, (place, "prompt"))
            close(feed(eng, 1, toks, [200, 213, 1]), want, kv, (place, "decoded"))


TILES = {
    # more gated rows, rows of the streams, columns of K and rows of the input product than one workgroup's share
    "gated": (model(attention(mlp=Y.clamped_mlp(14340)), width=64), (520, 300, 140)),
    "stream": (model(attention(mlp=Y.clamped_moe(3, 2, 30, shared=(52, 1.0))), width=8204, vocab=50), (300, 140, 20)),
    "columns": (model(attention(heads=16, kv_heads=4, dim=30, vdim=130, mlp=Y.clamped_mlp(4100)), delta(heads=32, kv_heads=2, dim=8, vdim=130, mlp=Y.clamped_moe(3, 2, 4100, shared=(4132, 2.0))),
                      width=132, vocab=50), (300, 140, 64, 30, 9)),
    "columns-odd": (model(attention(heads=16, kv_heads=4, dim=130, vdim=70, mlp=Y.clamped_mlp(4100)), delta(mlp=Y.clamped_moe(3, 2, 650, shared=(670, 2.0))), width=131, vocab=50), (300, 60, 9)),
    "shared": (model(attention(mlp=Y.clamped_moe(3, 2, 30, shared=(14340, 1.0))), width=64, vocab=30), (520,)),
    "experts": (model(attention(heads=2, kv_heads=2, mlp=Y.clamped_moe(8, 4, 1540, groups=(4, 3))), width=64, vocab=30), (1000,)),
    "heads": (model(attention(heads=120, kv_heads=60, dim=96, vdim=33), delta(heads=70, kv_heads=70, dim=16, vdim=16, decay_rank=300, gate_rank=530), width=64), (530, 200)),
}


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", sorted(TILES))
def test_products_of_every_tile_shape(tmp_path, name, kv):
    cfg, sizes = TILES[name]
    m = Vifanex(tmp_path / name, cfg, steer)
    with m.engine(kv, n_ctx=1152, n_batch=1024) as eng:
        for n in sizes:
            toks = m.tokens(n + 3, n)
            want = m.plain(toks)
            got = eng.step_logits([(0, toks[:n], 0)], [(0, k) for k in range(n)])
            close(got, want[:n], kv, n)
            close(feed(eng, 0, toks, [1], n), want[n:], kv, n)
            eng.seq_rm(0)


def sharpen(cfg, tensors):
    """Queries of every head point at the unrotated part of the key that token 7 leaves, far above all others."""
    m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    h = rms_norm(tensors["embed"], tensors["l0.norm1"], eps)
    for n in ("q", "k", "v"):
        tensors["l0.mix.%s.b" % n] *= 0.0
    for name in ("l0.hc1.in",):
        tensors[name] = np.full_like(tensors[name], 1.0 / cfg["streams"])
    k = tensors["l0.mix.k"] @ h[7]
    k = (k / np.sqrt((k * k).mean()) * tensors["l0.mix.k.norm"]).reshape(m["kv_heads"], m["dim"])
    k[:, :m["rot"]["dims"]] = 0
    k = np.repeat(k / np.sqrt((k * k).sum(1, keepdims=True)), m["heads"] // m["kv_heads"], 0)
    u = np.linalg.lstsq(h, np.ones(len(h)), rcond=None)[0]          # a constant part of the queries
    tensors["l0.mix.q"] = (0.02 * tensors["l0.mix.q"] + 4.0 * np.outer(k.ravel(), u)).astype(np.float32)
    tensors["l0.mix.q.norm"] = np.ones_like(tensors["l0.mix.q.norm"])


def edge_model(size, **kw):
    return model(attention(heads=4, kv_heads=2, dim=32, vdim=40, window=size, rot=Y.banded_rotary(8), scale=1.2, **kw), width=96, vocab=60, softcap=40.0)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("window", [31, 32, 33, 64, 97])
def test_window_edges(tmp_path, window, kv):
    """One key's score stands far out: it decides the output while its window lasts and not a token longer, in prompts,
    portions and decoding; windows are one page, one key to either side of one, and several pages. The plain statement
    with a window one key shorter or longer is far outside the limit at the edge."""
    m = Vifanex(tmp_path / ("edge%d" % window), edge_model(window), sharpen)
    for place in (0, 1, 5, 31, 32, 70):
        last = place + window - 1                                    # the last token that sees it
        toks = m.tokens(last + 5, place)
        toks[toks == 7] = 8
        toks[place] = 7
        want = m.plain(toks)
        for size, edge in ((window - 1, last), (window + 1, last + 1)):
            off = P.run_stack(edge_model(size), m.tensors, toks)[edge] - want[edge]
            assert np.sqrt((off * off).mean()) > 2 * LIMIT[kv] * np.sqrt((want * want).mean()), (window, place, size)
        with m.engine(kv, n_ctx=640) as eng:
            close(eng.step_logits([(0, toks, 0)], [(0, k) for k in range(len(toks))]), want, kv, (window, place, "prompt"))
            close(feed(eng, 1, toks, [last, 1]), want, kv, (window, place, "decoded"))
            close(feed(eng, 2, toks, [place + 1, max(last - place - 1, 2), 2]), want, kv, (window, place, "portions"))


@pytest.mark.parametrize("kv", KINDS)
def test_far_keys(tmp_path, kv):
    """A key hundreds of tokens back decides, at page borders and inside pages; without it the output is another."""
    m = Vifanex(tmp_path / "far", edge_model(700), sharpen)
    for place in (0, 31, 32, 100):
        toks = m.tokens(620, place)
        toks[toks == 7] = 8
        without = P.run_stack(m.cfg, m.tensors, toks)[-8:]
        toks[place] = 7
        want = m.plain(toks)
        off = without - want[-8:]
        assert np.sqrt((off * off).mean(1)).min() > 2 * LIMIT[kv] * np.sqrt((want * want).mean())
        with m.engine(kv, n_ctx=2048, n_batch=640) as eng:
            close(eng.step_logits([(0, toks, 0)], [(0, k) for k in range(620)]), want, kv, (place, "prompt"))
            close(feed(eng, 1, toks, [300, 312, 1]), want, kv, (place, "decoded"))


@pytest.mark.parametrize("kv", KINDS)
def test_long_decoding(models, kv):
    m = models("all")
    toks = m.tokens(420, 77)
    with m.engine(kv) as eng:
        close(feed(eng, 3, toks, [20, 1]), m.plain(toks), kv)


@pytest.mark.parametrize("kv", KINDS)
def test_long_prompts(models, kv):
    m = models("wide")
    toks, other = m.tokens(400, 78), m.tokens(70, 79)
    with m.engine(kv, n_ctx=1024, n_batch=512) as eng:
        close(feed(eng, 0, toks, [400]), m.plain(toks), kv)
        close(feed(eng, 1, toks, [129, 200, 3]), m.plain(toks), kv)
        eng.seq_rm(1)
        got = eng.step_logits([(1, toks[:300], 0), (2, other, 0), (3, other[:1], 0)], [(0, 299), (1, 69), (2, 0)])
        close(got, np.stack([m.plain(toks)[299], m.plain(other)[69], m.plain(other)[0]]), kv)


@pytest.mark.parametrize("kv", KINDS)
def test_copies_and_snapshots(models, kv):
    m = models("all")
    toks, tail = m.tokens(100, 4), m.tokens(40, 6)
    longer = np.concatenate([toks, tail])
    with m.engine(kv, n_ctx=1024) as eng:
        assert eng.is_hybrid()
        feed(eng, 0, toks, [100])
        eng.seq_cp(0, 1)
        close(feed(eng, 1, longer, [3, 1, 36], 100), m.plain(longer)[100:], kv)
        saved = eng.seq_save(0)
        eng.seq_rm(0)
        eng.seq_load(2, saved)
        close(feed(eng, 2, longer, [40], 100), m.plain(longer)[100:], kv)
        with pytest.raises(E.EngineError, match="partial"):
            eng.seq_rm(2, 50, -1)


@pytest.mark.parametrize("kv", KINDS)
def test_copies_of_attention_only_models(models, kv):
    m = models("values-mixed")
    toks, tail = m.tokens(100, 4), m.tokens(40, 6)
    with m.engine(kv, n_ctx=1024) as eng:
        assert not eng.is_hybrid()
        feed(eng, 0, toks, [100])
        eng.seq_cp(0, 1, 0, 70)                               # shares pages, then writes into a shared one
        mixed = np.concatenate([toks[:70], tail])
        close(feed(eng, 1, mixed, [3, 1, 20], 70), m.plain(mixed)[70:], kv)
        eng.seq_rm(0, 50, -1)
        mixed = np.concatenate([toks[:50], tail])
        close(feed(eng, 0, mixed, [17], 50), m.plain(mixed)[50:], kv)


def test_greedy_generation_through_scheduler_and_generators(tmp_path):
    m = Model(tmp_path / "greedy", CONFIGS["all"], decide_routing)
    prompts = [list(map(int, m.tokens(n, 40 + n))) for n in (70, 9, 33, 1)]
    prompts.append(prompts[0] + list(map(int, m.tokens(4, 1))))        # extends a finished prompt
    n_new = [12, 20, 6, 15, 8]
    expect = [plain_greedy(m, p, n) for p, n in zip(prompts, n_new)]
    assert all(lead > 1e-3 for _, lead in expect), "the prompts of this test leave ties"
    assert sum(len(set(toks)) > 3 for toks, _ in expect) >= 4
    with m.engine(E.KV_F32, n_ctx=1024, n_batch=64) as eng:
        sched = S.Scheduler.over_engine(eng, S.SchedulerOptions(mode=S.CONTINUOUS, n_batch=64, queue_capacity=32, event_capacity=256,
                                                                slow_client_timeout=1.0, prefix_cache=True, min_prefix_len=4,
                                                                swap_min_tokens=1 << 62))
        sched.initialize()
        for wave in ([0, 1, 2, 3], [4], [1]):
            streams = [(i, sched.submit(S.Request.single(prompts[i], E.SamplingParamsV2.greedy(max_new_tokens=n_new[i])))) for i in wave]
            sched.run_until_idle()
            for i, st in streams:
                toks = [ev.token for ev in st.drain() if ev.type == "Token"]
                assert toks == expect[i][0], i
        sched.close()
    with m.engine(E.KV_F32, n_ctx=1024, n_batch=64) as eng:
        greedy = lambda n: (1e-4, 1.0, n, 1)               # the v1 sampler at a temperature that leaves only the best
        got = eng.generate_continuous([(p, greedy(n)) for p, n in zip(prompts[:4], n_new)])
        assert [g[0] for g in got] == [e[0] for e in expect[:4]]
        got = eng.generate_continuous([(prompts[4], greedy(n_new[4]))])
        assert got[0][0] == expect[4][0]
        got = eng.generate_batch(prompts[2], [greedy(n_new[2])] * 3)
        assert all(g[0] == expect[2][0] for g in got)


@pytest.mark.parametrize("dtype, kv", [("float32", E.KV_F32), ("bfloat16", E.KV_F16)])
def test_trace_replay(models, tmp_path, capsys, monkeypatch, dtype, kv):
    from retrograd_amd import trace_replay

    m = models("all")
    a, b = m.tokens(60, 1), m.tokens(20, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:33].tolist(), "want": [0, 32]}, {"id": "b", "tokens": b.tolist(), "want": [19]}], "end": ["b"]},
             {"step": 1, "entries": [{"id": "a", "tokens": a[33:34].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "c", "tokens": b.tolist(), "want": [3]}, {"id": "a", "tokens": a[34:].tolist(), "want": [25]}], "end": ["a", "c"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    assert trace_replay.main(["--model", str(m.folder), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "128"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    read = lambda n: np.fromfile(tmp_path / ("%d.f32" % n), "<f4").reshape(-1, m.cfg["vocab"])
    close(read(0), np.stack([m.plain(a)[0], m.plain(a)[32], m.plain(b)[19]]), kv)
    assert not (tmp_path / "1.f32").exists()
    close(read(2), np.stack([m.plain(b)[3], m.plain(a)[59]]), kv)


def test_refusals(models, tmp_path):
    m = models("all")
    base = dict(n_ctx=256, n_seq_max=2, n_batch=64, n_ubatch=64)
    for i, (name, edit) in enumerate({"l0.mix.a1": lambda t: t.pop("l0.mix.a1"), "l0.mix.g2": lambda t: t.update({"l0.mix.g2": t["l0.mix.g2"][:, :-1]}),
                                      "l1.mix.v.b": lambda t: t.pop("l1.mix.v.b"), "l3.hc2.mix": lambda t: t.update({"l3.hc2.mix": t["l3.hc2.mix"][:2]}),
                                      "head": lambda t: t.pop("head"), "l0.mlp.e5.down": lambda t: t.pop("l0.mlp.e5.down")}.items()):
        t = dict(m.tensors)
        edit(t)
        with pytest.raises(E.EngineError, match=name):
            E.Engine(Y.write_checkpoint(tmp_path / str(i), m.cfg, t), E.EngineConfig(**base))
