"""The Kilurax design through the engine against the plain statements in plain_kilurax.py: attention and Mamba-2 side by side,
linear attention with a forget gate, the gated delta rule with a decay per head, grouped norms around every sublayer, the
convolution of what a sublayer reads, the embedding of neighbouring tokens, experts whose scores weigh their inputs. Every
mechanism alone and together, prompts against decoding and portions, batches, reused pages and slots."""
import io
import json

import numpy as np
import pytest

import plain_kilurax as P
from retrograd_amd import engine as E
from retrograd_amd import scheduler as S
from retrograd_amd import synth_stack as Y
from stack_helpers import KINDS, LIMIT, Model, close, feed, plain_greedy

pytestmark = pytest.mark.gpu

ROT = Y.rotary(12, 500.0)


def both(attention=(6, 2, 20, 28), mamba2=(4, 9, 12, 2, 3, 2), scales=(0.8, 1.3), rot=ROT, mlp=None, **kw):
    return Y.parallel_mixer_layer(attention, mamba2, scales, rot, mlp, **kw)


def forget(heads=3, dim=20, vdim=28, mlp=None):
    return Y.hgrn2_layer(heads, dim, vdim, mlp)


def delta(heads=4, kv_heads=2, dim=20, vdim=24, conv=3, mlp=None):
    return Y.delta_layer(heads, kv_heads, dim, vdim, conv, mlp)


def model(*layers, width=72, vocab=40, **kw):
    return Y.kilurax(width, vocab, list(layers), **kw)


CONFIGS = {
    # each mechanism alone
    "side-by-side": model(both()),
    "attention": model(both(scales=(1.0, 0.0))),
    "attention-own-keys": model(both((3, 3, 24, 24), scales=(-0.7, 0.0), rot=Y.rotary(24), scale=0.9)),
    "rotary-partial": model(both(rot=Y.rotary(8, 300.0), scales=(1.0, 0.1))),
    "rotary-none": model(both(rot=Y.rotary(0), scales=(1.0, 0.1))),
    "rotary-absent": model(both(rot=None, scales=(1.0, 0.1))),
    "values-narrow": model(both((6, 3, 66, 9), scales=(1.0, 0.1))),
    "values-wide": model(both((4, 1, 7, 50), rot=Y.rotary(6), scales=(1.0, 0.1))),
    "mamba2": model(both(scales=(0.0, 1.0))),
    "mamba2-one-group": model(both(mamba2=(5, 8, 40, 1, 4, 1), scales=(0.0, 1.0))),
    "mamba2-group-each": model(both(mamba2=(6, 10, 7, 6, 2, 5), scales=(0.0, 1.0))),
    "mamba2-no-convolution": model(both(mamba2=(4, 9, 12, 2, 1, 3), scales=(0.1, 1.0))),
    "mamba2-long-taps": model(both(mamba2=(4, 9, 12, 2, 7, 2), scales=(0.1, 1.0))),
    "forget": model(forget()),
    "forget-one-head": model(forget(heads=1, dim=33, vdim=7)),
    "forget-many-heads": model(forget(heads=11, dim=6, vdim=10)),
    "delta": model(delta()),
    "delta-shared-keys": model(delta(heads=6, kv_heads=1)),
    "delta-own-keys": model(delta(heads=3, kv_heads=3, conv=4)),
    "delta-no-convolution": model(delta(conv=1)),
    "delta-two-taps": model(delta(conv=2)),
    "delta-long-taps": model(delta(conv=6)),
    "one-norm-group": model(forget(), groups=1),
    "odd-norm-groups": model(forget(), groups=8),
    "norm-group-each": model(delta(), groups=72, taps=2, eps=0.1),
    "odd-width": model(forget(), delta(), width=75, groups=5),
    "input-of-own-token": model(forget(), delta(), taps=1),
    "input-two-taps": model(forget(), delta(), taps=2),
    "input-four-taps": model(forget(), delta(), taps=4),
    "input-many-taps": model(forget(), both(), taps=9),
    "pairs-one-bucket": model(forget(), pairs=(1, 3, 4)),
    "pairs-own-row": model(forget(), pairs=(1600, 40, 1)),
    "pairs-large-factors": model(forget(), pairs=(211, (1 << 52) + 12345, (1 << 40) + 77)),
    "pairs-previous-only": model(forget(), pairs=(41, 1, 0)),
    "residual-whole": model(delta(), forget(), residual=1.0),
    "experts": model(forget(mlp=Y.moe_mlp(6, 2, 40))),
    "experts-shared": model(delta(mlp=Y.moe_mlp(6, 3, 20, 50))),
    "experts-top-one": model(forget(mlp=Y.moe_mlp(5, 1, 30, 33))),
    "experts-all": model(forget(mlp=Y.moe_mlp(3, 3, 24, 20))),
    "experts-many": model(forget(mlp=Y.moe_mlp(300, 5, 9, 33))),
    "experts-one": model(forget(mlp=Y.moe_mlp(1, 1, 30))),
    # together, every layer of other sizes; the width is no multiple of a tile
    "all": model(
        delta(mlp=Y.moe_mlp(8, 2, 33, 41)),
        both(mlp=Y.moe_mlp(5, 1, 20)),
        forget(heads=5, dim=37, vdim=11),
        both((3, 3, 40, 17), (10, 6, 33, 5, 4, 3), (1.2, 0.4), Y.rotary(40, 300.0), scale=0.5),
        forget(heads=2, dim=70, vdim=50, mlp=Y.moe_mlp(9, 3, 50, 20)),
        delta(heads=10, kv_heads=5, dim=70, vdim=34, conv=2),
        both((8, 1, 18, 56), (1, 30, 20, 1, 5, 2), (0.3, -0.9), Y.rotary(18, 90.0)),
        width=105, vocab=50, groups=3, taps=4, residual=0.4, eps=1e-4, embedding_scale=3.0, pairs=(307, 11, 101)),
    # sizes of one (a norm of one value is its sign but for eps)
    "ones": model(
        both((1, 1, 1, 1), (1, 1, 1, 1, 1, 1), (1.0, 1.0), Y.rotary(0), mlp=Y.moe_mlp(1, 1, 1, 1), scale=1.5),
        forget(heads=1, dim=1, vdim=1), delta(heads=1, kv_heads=1, dim=1, vdim=1, conv=1),
        both((2, 1, 2, 1), (2, 1, 2, 1, 2, 1), (0.5, 0.5), Y.rotary(2, 7.0)), width=9, vocab=5, groups=1, taps=2, pairs=(2, 1, 1), eps=0.3),
    # sizes of a real model's heads and experts
    "wide": model(
        delta(heads=8, kv_heads=4, dim=128, vdim=128, conv=4, mlp=Y.moe_mlp(16, 4, 512, 544)),
        both((16, 4, 128, 128), (16, 64, 128, 4, 4, 4), (0.7, 0.6), Y.rotary(128, 1e5), mlp=Y.moe_mlp(12, 3, 160)),
        forget(heads=6, dim=96, vdim=200, mlp=Y.moe_mlp(12, 2, 160, 96)),
        both((20, 20, 72, 56), (8, 24, 40, 1, 4, 1), (1.0, 1.0), Y.rotary(72, 1e4)),
        forget(heads=4, dim=128, vdim=128), width=512, vocab=150, groups=4, taps=4, embedding_scale=2.0, pairs=(1009, 3, 17)),
}
BIG = ["all", "ones", "wide"]


def steer(cfg, tensors):
    """Routing decided by the token, so that rounding chooses no other expert (a test of rounding must not rest on a close
    call): the embedding outweighs what is added to it and what the convolution brings, the routers' chosen logits stand
    clear of the others, and the scores are far from one."""
    routed = [i for i, layer in enumerate(cfg["layers"]) if layer.get("mlp")]
    if not routed:
        return
    rng = np.random.default_rng(1)
    tensors["bigram"] *= 0.05 * cfg["embedding"]["scale"]
    tensors["embed.norm"] = 1.0 + 0.1 * tensors["embed.norm"]
    for name in tensors:
        if name.endswith("b") and ".norm" in name:
            tensors[name] *= 0.15
        elif name.endswith("canon2"):
            tensors[name] *= 0.1
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = P.grouped_norm(tensors["embed"] * cfg["embedding"]["scale"], tensors["embed.norm"], eps, groups)
    for i in routed:
        n, top = cfg["layers"][i]["mlp"]["router"]["experts"], cfg["layers"][i]["mlp"]["router"]["top"]
        h = P.grouped_norm(x, tensors["l%d.norm2" % i], eps, groups) * (1 + tensors["l%d.canon2" % i][:, -1])
        z = rng.uniform(-9.0, -6.0, (cfg["vocab"], n))
        for row in z:
            row[rng.permutation(n)[:top]] = rng.uniform(-0.7, 1.2, top)
        tensors["l%d.mlp.router" % i] = np.linalg.lstsq(h, z, rcond=None)[0].T.astype(np.float32)


class Kilurax(Model):
    """Its plain statement also makes sure that the routing is decided."""
    def plain(self, tokens):
        key = tuple(int(t) for t in tokens)
        if key not in self.seen:
            leads = []
            self.seen[key] = P.run_stack(self.cfg, self.tensors, tokens, leads=leads)
            assert all(lead.min() > 0.2 for lead in leads), [float(lead.min()) for lead in leads]
        return self.seen[key]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Kilurax(tmp_path_factory.mktemp("kilurax") / name, CONFIGS[name], steer)
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
@pytest.mark.parametrize("name", BIG + ["side-by-side", "mamba2-long-taps", "forget", "delta", "delta-long-taps", "input-many-taps", "input-of-own-token", "pairs-previous-only", "odd-norm-groups", "experts-top-one"])
def test_token_by_token_is_the_prompt(models, name, kv):
    m = models(name)
    toks = m.tokens(130)
    with m.engine(kv) as eng:
        close(feed(eng, 1, toks, [1]), m.plain(toks), kv)
        eng.seq_rm(1)
        close(feed(eng, 2, toks, [77, 1]), m.plain(toks), kv)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", BIG + ["input-many-taps", "delta-no-convolution"])
def test_portions_of_any_size(models, name, kv):
    m = models(name)
    toks = m.tokens(150)
    with m.engine(kv) as eng:
        for sizes in ([2], [3], [7, 2, 31, 5], [16], [32], [33, 31, 2], [64, 65], [128, 2], [149, 1]):
            close(feed(eng, 0, toks, sizes), m.plain(toks), kv, sizes)
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", ["all", "wide", "input-many-taps"])
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
@pytest.mark.parametrize("dim, vdim", [(6, 30), (96, 20), (60, 90), (50, 100), (120, 40), (160, 128), (200, 66), (256, 256), (270, 90), (40, 300)])
def test_key_and_value_widths(tmp_path, dim, vdim, kv):
    """Pairs of widths the attention kernels are compiled for, rounded up to and beyond them, with few, some and many query
    heads per key head: whole prompts, decoding one sequence (whose keys are shared out) and many."""
    for heads, kv_heads in ((5, 5), (40, 2), (20, 1)):
        m = Kilurax(tmp_path / ("d%dh%dg%d" % (dim, heads, kv_heads)), model(
            both((heads, kv_heads, dim, vdim), (1, 4, 4, 1, 2, 1), (1.0, 0.1), Y.rotary(dim // 4 * 2), scale=2 * dim ** -0.5), width=48, vocab=60))
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
    """Every shape of the recurrences' kernels: heads too wide for the chunks or for one block of columns among them."""
    m = Kilurax(tmp_path / "state", model(delta(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=4), forget(heads=heads, dim=dim, vdim=vdim), width=60, vocab=50, eps=0.01))
    toks = m.tokens(200, dim)
    want = m.plain(toks)
    with m.engine(kv) as eng:
        for sizes in ([200], [1], [70, 3, 1, 32, 31]):
            close(feed(eng, 0, toks, sizes), want, kv, sizes)
            eng.seq_rm(0)


def spread(**ranges):
    """Tensors by the ends of their names, spread over a range in mixed order."""
    def edit(cfg, tensors):
        for name in tensors:
            for end, ends in ranges.items():
                if name.endswith("." + end.replace("f_b", "f.b")):
                    v = np.linspace(*ends, tensors[name].size).astype(np.float32)
                    tensors[name] = v[np.random.default_rng(len(name)).permutation(v.size)].reshape(tensors[name].shape)
    return edit


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name, ranges", [
    ("none", dict(A_log=(-12.0, -9.0), dt_bias=(-6.0, -4.0), f_b=(8.0, 14.0), lower=(0.9, 1.0))),
    ("all", dict(A_log=(2.0, 4.0), dt_bias=(-1.0, 6.0), f_b=(-30.0, -3.0), lower=(0.0, 0.0))),
    ("both", dict(A_log=(-5.0, 3.0), dt_bias=(-8.0, 5.0), f_b=(-12.0, 12.0), lower=(0.0, 1.0)))])
def test_weak_and_strong_decays(tmp_path, name, ranges, kv):
    """States that forget nothing over the whole prompt beside such that forget everything at every token."""
    for i, layer in enumerate((delta(heads=4, kv_heads=2, dim=48, vdim=32), forget(heads=2, dim=48, vdim=40), both(mamba2=(6, 12, 20, 3, 3, 1), scales=(0.2, 1.0)))):
        m = Kilurax(tmp_path / (name + str(i)), model(layer, residual=1.0), spread(**ranges))
        toks = m.tokens(300, 1)
        want = m.plain(toks)
        with m.engine(kv, n_batch=320) as eng:
            for sizes in ([300], [1], [100, 33, 2]):
                close(feed(eng, 0, toks, sizes), want, kv, (i, name, sizes))
                eng.seq_rm(0)


def column_per_token(cfg, tensors):
    """Every token has a column of its own, and neither pairs nor neighbours add anything."""
    e = np.zeros((cfg["vocab"], cfg["width"]), np.float32)
    e[np.arange(cfg["vocab"]), np.arange(cfg["vocab"])] = 1.0
    tensors["embed"], tensors["bigram"] = e, 0.0 * tensors["bigram"]
    for name in tensors:
        if ".canon" in name:
            tensors[name] = 0.0 * tensors[name]


def far_delta(cfg, tensors):
    """Token 7 alone writes to key channel 0, which every query reads and nothing decays."""
    spread(A_log=(-9.0, -8.0), dt_bias=(-6.0, -5.0))(cfg, tensors)
    column_per_token(cfg, tensors)
    for n in ("q", "k", "v"):
        taps = np.zeros_like(tensors["l0.mix.%s.conv" % n])
        taps[:, -1] = 1.0
        tensors["l0.mix.%s.conv" % n] = taps
    D, n = cfg["layers"][0]["mixer"]["dim"], cfg["vocab"]
    k, q = np.zeros((D, cfg["width"])), np.zeros((D, cfg["width"]))
    k[1:, :n] = np.random.default_rng(2).uniform(0.5, 1.0, (D - 1, n))
    k[0, :n] = -12.0                                    # SiLU closes the channel for every other token
    k[:, 7] = 0.0
    k[0, 7] = 1.0
    q[0] = 1.0
    q[1:] = -12.0
    tensors["l0.mix.k"], tensors["l0.mix.q"] = (4.0 * k).astype(np.float32), (4.0 * q).astype(np.float32)


def far_forget(cfg, tensors):
    """Token 7 alone opens channel 0, which every query reads; for all others its gate keeps what it holds."""
    column_per_token(cfg, tensors)
    D, n = cfg["layers"][0]["mixer"]["dim"], cfg["vocab"]
    f, q = np.zeros((D, cfg["width"])), np.zeros((D, cfg["width"]))
    f[0, :n] = 8.0
    f[0, 7] = -4.0
    q[0, :n] = 4.0
    q[1:, :n] = -12.0
    tensors["l0.mix.f"], tensors["l0.mix.q"] = f.astype(np.float32), q.astype(np.float32)
    tensors["l0.mix.f.b"], tensors["l0.mix.lower"] = 0.0 * tensors["l0.mix.f.b"], 0.0 * tensors["l0.mix.lower"]


def far_space(cfg, tensors):
    """Token 7 alone has a large step, in a state that decays slowly."""
    column_per_token(cfg, tensors)
    m, n = cfg["layers"][0]["mixer"]["right"], cfg["vocab"]
    r = "l0.mix.right."
    inner, N = m["heads"] * m["vdim"], m["state"] * m["groups"]
    w = 0.3 * tensors[r + "in"]
    w[-m["heads"]:] = 0.0
    w[-m["heads"]:, 7] = 3.0
    w[2 * inner:2 * inner + 2 * N, :n] = 1.0                                    # every token writes and reads the same direction
    tensors[r + "in"] = w
    tensors[r + "conv"] = np.zeros_like(tensors[r + "conv"])
    tensors[r + "conv"][:, -1] = 1.0
    tensors[r + "A_log"], tensors[r + "dt_bias"] = np.full(m["heads"], -7.0, np.float32), np.full(m["heads"], -5.0, np.float32)


def far_key(cfg, tensors):
    """Every query points at the unrotated part of the key that token 7 leaves, far above all others."""
    column_per_token(cfg, tensors)
    m, n = cfg["layers"][0]["mixer"]["left"], cfg["vocab"]
    a = "l0.mix.left."
    k, q = np.zeros((m["kv_heads"], m["dim"], cfg["width"])), np.zeros((m["heads"], m["dim"], cfg["width"]))
    k[:, -1, 7] = 3.0
    q[:, -1, :n] = 3.0
    tensors[a + "k"] = (k.reshape(-1, cfg["width"]) + 0.02 * tensors[a + "k"]).astype(np.float32)
    tensors[a + "q"] = (q.reshape(-1, cfg["width"]) + 0.02 * tensors[a + "q"]).astype(np.float32)
    for name in ("q.b", "k.b"):
        tensors[a + name] *= 0.0


FAR = {"delta": (delta(heads=1, kv_heads=1, dim=16, vdim=24), far_delta), "forget": (forget(heads=1, dim=16, vdim=24), far_forget),
       "space": (both((1, 1, 4, 4), (2, 10, 8, 1, 2, 1), (0.0, 1.0), Y.rotary(4)), far_space),
       "key": (both((4, 2, 32, 40), (1, 4, 4, 1, 2, 1), (1.0, 0.0), Y.rotary(8), scale=1.2), far_key)}


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("kind", sorted(FAR))
def test_what_one_token_left_decides_far_away(tmp_path, kind, kv):
    """One token stands out and decides what hundreds of later tokens read, across chunks, pages, steps and decoding; without
    it the output is another."""
    layer, edit = FAR[kind]
    m = Kilurax(tmp_path / "far", model(layer, width=60, vocab=50, residual=1.0), edit)
    for place in (0, 31, 32, 63, 64, 100):
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


def only_neighbours(cfg, tensors):
    """Sublayers read nothing but the token furthest back."""
    for name in tensors:
        if ".canon" in name:
            tensors[name] = 0.1 * tensors[name]
            tensors[name][:, 0] = 2.5


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("taps", [2, 3, 4, 6])
def test_reach_of_the_input_convolution(tmp_path, taps, kv):
    """The oldest tap outweighs the others; with one tap fewer the output is far outside the limit. The start of a portion,
    portions shorter than the taps, single tokens and several sequences at once."""
    m = Kilurax(tmp_path / "reach", model(forget(), delta(), taps=taps), only_neighbours)
    toks, other = m.tokens(50, taps), m.tokens(31, 90)
    want = m.plain(toks)
    short = {k: v[:, 1:] if ".canon" in k else v for k, v in m.tensors.items()}
    off = P.run_stack(dict(m.cfg, canon={"taps": taps - 1}), short, toks)[taps:] - want[taps:]
    assert np.sqrt((off * off).mean(1)).min() > 2 * LIMIT[kv] * np.sqrt((want * want).mean())
    with m.engine(kv) as eng:
        for sizes in ([50], [1], [2], [3, 1, 5], [taps - 1], [taps, 1, 1, 2]):
            close(feed(eng, 0, toks, sizes), want, kv, sizes)
            eng.seq_rm(0)
        for at in range(31):                                        # single tokens of two sequences, then a portion beside one
            got = eng.step_logits([(1, toks[at:at + 1], at), (3, other[at:at + 1], at)], [(0, 0), (1, 0)])
            close(got, np.stack([want[at], m.plain(other)[at]]), kv, at)
        got = eng.step_logits([(3, toks[:1], 31), (1, toks[31:], 31)], [(1, k) for k in range(19)])
        close(got, want[31:], kv)


@pytest.mark.parametrize("kv", KINDS)
def test_the_pair_embedding_alone_tells_tokens_apart(tmp_path, kv):
    """Tokens embedded alike: only the row of each pair, and that of the first token, is left. Sequences that start anew in a
    used slot, portions and decoding."""
    def edit(cfg, tensors):
        tensors["embed"][:] = tensors["embed"][0]
        tensors["bigram"] *= 3.0
    m = Kilurax(tmp_path / "pairs", model(forget(), vocab=12, pairs=(53, 17, 4)), edit)
    a, b = m.tokens(60, 1), m.tokens(45, 2)
    with m.engine(kv, slots=2) as eng:
        for toks in (a, b, a[::-1]):
            for sizes in ([60], [1], [2], [13, 1, 1, 3]):
                close(feed(eng, 1, toks, sizes), m.plain(toks), kv, sizes)
                eng.seq_rm(1)


TILES = {
    # more expert rows, rows of the stream, columns of K and rows of the input product than one workgroup's share
    "stream": (model(forget(mlp=Y.moe_mlp(3, 2, 30, 52)), width=8208, vocab=50, groups=3), (300, 140, 20)),
    "stream-odd": (model(forget(), width=4203, vocab=50, groups=3), (300, 20)),
    "columns": (model(both((16, 4, 30, 130), (40, 33, 8, 1, 2, 1), (1.0, 0.7)), delta(heads=32, kv_heads=2, dim=8, vdim=130, mlp=Y.moe_mlp(3, 2, 4100, 4132)),
                      forget(heads=33, dim=4, vdim=130), width=132, vocab=50), (300, 140, 64, 30, 9)),
    "columns-odd": (model(both((16, 4, 130, 70), (7, 9, 5, 1, 2, 3), (1.0, 0.7)), delta(mlp=Y.moe_mlp(3, 2, 650, 670)), width=131, vocab=50, groups=1), (300, 60, 9)),
    "shared": (model(forget(mlp=Y.moe_mlp(3, 2, 30, 14340)), width=64, vocab=30), (520,)),
    "experts": (model(forget(mlp=Y.moe_mlp(8, 4, 1540)), width=64, vocab=30), (1000,)),
    "heads": (model(both((120, 60, 96, 33), (70, 16, 16, 7, 3, 10), (1.0, 1.0)), delta(heads=70, kv_heads=70, dim=16, vdim=16), forget(heads=90, dim=16, vdim=16), width=64), (530, 200)),
}


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", sorted(TILES))
def test_products_of_every_tile_shape(tmp_path, name, kv):
    cfg, sizes = TILES[name]
    m = Kilurax(tmp_path / name, cfg, steer)
    with m.engine(kv, n_ctx=1152, n_batch=1024) as eng:
        for n in sizes:
            toks = m.tokens(n + 3, n)
            want = m.plain(toks)
            got = eng.step_logits([(0, toks[:n], 0)], [(0, k) for k in range(n)])
            close(got, want[:n], kv, n)
            close(feed(eng, 0, toks, [1], n), want[n:], kv, n)
            eng.seq_rm(0)


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
        for first in ([100], [99, 1]):                        # leaves what the next step remembers in either plane
            feed(eng, 0, toks, first)
            eng.seq_cp(0, 1)
            close(feed(eng, 1, longer, [3, 1, 36], 100), m.plain(longer)[100:], kv)
            saved = eng.seq_save(0)
            eng.seq_rm(0)
            eng.seq_load(2, saved)
            close(feed(eng, 2, longer, [1, 39], 100), m.plain(longer)[100:], kv)
            with pytest.raises(E.EngineError, match="partial"):
                eng.seq_rm(2, 50, -1)
            for slot in (1, 2):
                eng.seq_rm(slot)


def test_greedy_generation_through_scheduler_and_generators(models):
    m = models("all")
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
    edits = {"bigram": lambda t: t.update(bigram=t["bigram"][:-1]), "embed.norm": lambda t: t.pop("embed.norm"), "l0.norm2b": lambda t: t.pop("l0.norm2b"),
             "l0.canon1": lambda t: t.update({"l0.canon1": t["l0.canon1"][:, 1:]}), "l0.mix.a": lambda t: t.pop("l0.mix.a"),
             "l1.mix.left.o.b": lambda t: t.pop("l1.mix.left.o.b"), "l1.mix.right.in": lambda t: t.update({"l1.mix.right.in": t["l1.mix.right.in"][1:]}),
             "l2.mix.lower": lambda t: t.update({"l2.mix.lower": t["l2.mix.lower"] - 2}), "head": lambda t: t.pop("head"), "l0.mlp.e5.down": lambda t: t.pop("l0.mlp.e5.down")}
    for i, (name, edit) in enumerate(edits.items()):
        t = dict(m.tensors)
        edit(t)
        with pytest.raises(E.EngineError, match=name):
            E.Engine(Y.write_checkpoint(tmp_path / str(i), m.cfg, t), E.EngineConfig(**base))
