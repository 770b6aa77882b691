"""The Pomisun design through the engine against the plain statements in plain_pomisun.py: grouped attention whose values
are its keys, in chunks, with stretched rotary positions and soft-capped scores; gated and expert feed-forwards; looped
layers. Every mechanism alone and together, prompts against decoding and portions, batches, reused pages and slots."""
import io
import json

import numpy as np
import pytest

import plain_pomisun as P
from retrograd_amd import engine as E
from retrograd_amd import scheduler as S
from retrograd_amd import synth_stack as Y
from stack_helpers import KINDS, LIMIT, Model, close, feed, plain_greedy

pytestmark = pytest.mark.gpu


def attention(heads=6, kv_heads=2, dim=24, mask=45, rot=None, mlp=None, **kw):
    return Y.attention_layer(heads, kv_heads, dim, mask, rot or Y.rotary(16, 1000.0, factor=8.0, original=40, fast=8.0, slow=0.5), mlp, **kw)


def one_layer(**kw):
    return Y.pomisun(72, 40, [attention(**kw)])


CONFIGS = {
    # each mechanism alone
    "attention": one_layer(rot=Y.rotary(24)),
    "attention-unbounded": one_layer(rot=Y.rotary(24), mask=1 << 20),
    "rotary-partial": one_layer(rot=Y.rotary(10, 500.0)),
    "rotary-none": one_layer(rot=Y.rotary(0)),
    "rotary-stretched": one_layer(),
    "softcap": one_layer(softcap=1.3, scale=0.7),
    "dense": one_layer(mlp=Y.dense_mlp(50)),
    "experts": one_layer(mlp=Y.moe_mlp(6, 2, 40)),
    "experts-shared": one_layer(mlp=Y.moe_mlp(6, 3, 20, 50)),
    "experts-all": one_layer(mlp=Y.moe_mlp(3, 3, 24, 20)),
    "experts-many": one_layer(mlp=Y.moe_mlp(300, 5, 9, 33)),
    "experts-one": one_layer(mlp=Y.moe_mlp(1, 1, 30)),
    "loop": Y.pomisun(72, 40, [attention(mlp=Y.dense_mlp(40)), attention(mask=20)], loop=(0, 1, 3)),
    "loop-all": Y.pomisun(72, 40, [attention(), attention(mask=20)], loop=(0, 2, 2)),
    "loop-once": Y.pomisun(72, 40, [attention(), attention(mask=20)], loop=(1, 2, 1)),
    # together, every layer of other sizes; the width is no multiple of a tile
    "all": Y.pomisun(107, 50, [
        attention(mlp=Y.moe_mlp(7, 2, 33, 41), softcap=2.0),
        attention(heads=3, kv_heads=3, dim=40, mask=33, rot=Y.rotary(40, 300.0), mlp=Y.dense_mlp(90)),
        attention(heads=8, kv_heads=1, dim=18, mask=70, mlp=Y.moe_mlp(4, 3, 20), softcap=5.0, scale=0.5),
        attention(heads=5, kv_heads=5, dim=32, mask=9),
        attention(heads=4, kv_heads=2, dim=66, mask=64, rot=Y.rotary(22, 90.0, factor=2.0, original=30), mlp=Y.moe_mlp(9, 1, 50, 20))],
        eps=1e-4, loop=(1, 4, 2)),
    # sizes of one
    "ones": Y.pomisun(9, 5, [
        attention(heads=1, kv_heads=1, dim=1, mask=1, rot=Y.rotary(0), mlp=Y.moe_mlp(1, 1, 1, 1), scale=1.5),
        attention(heads=2, kv_heads=1, dim=2, mask=2, rot=Y.rotary(2, 7.0), mlp=Y.dense_mlp(1))], loop=(0, 1, 2)),
    # sizes of a real model's heads and experts
    "wide": Y.pomisun(512, 150, [
        attention(heads=16, kv_heads=4, dim=128, mask=100, rot=Y.rotary(128, 1e5, factor=4.0, original=64), mlp=Y.dense_mlp(1536), softcap=30.0),
        attention(heads=40, kv_heads=1, dim=64, mask=150, rot=Y.rotary(32, 1e4), mlp=Y.moe_mlp(16, 4, 512, 544), softcap=8.0),
        attention(heads=8, kv_heads=8, dim=64, mask=64, rot=Y.rotary(64), mlp=Y.moe_mlp(12, 3, 160))], loop=(0, 2, 2)),
}
BIG = ["all", "ones", "wide"]


def decide_routing(cfg, tensors):
    """Routers that follow the token: its chosen experts' logits stand clear of the others', so that rounding chooses
    no other expert (a test of rounding must not rest on a close call)."""
    rng = np.random.default_rng(1)
    tensors["embed"] = 5.0 * tensors["embed"]
    for i, layer in enumerate(cfg["layers"]):
        if not layer.get("mlp") or layer["mlp"]["kind"] != "moe":
            continue
        n, top = layer["mlp"]["router"]["experts"], layer["mlp"]["router"]["top"]
        h = P.rms_norm_around_one(tensors["embed"], tensors["l%d.norm2" % i], cfg["norm"]["eps"])
        z = rng.uniform(-1.0, 1.0, (cfg["vocab"], n))
        for row in z:
            row[rng.permutation(n)[:top]] += 7.0
        tensors["l%d.mlp.router" % i] = np.linalg.lstsq(h, z, rcond=None)[0].T.astype(np.float32)


class Pomisun(Model):
    """Its plain statement also makes sure that the routing is decided."""
    def plain(self, tokens):
        key = tuple(int(t) for t in tokens)
        if key not in self.seen:
            leads = []
            self.seen[key] = P.run_stack(self.cfg, self.tensors, tokens, leads=leads)
            assert all(lead.min() > 0.05 for lead in leads), [float(lead.min()) for lead in leads]
        return self.seen[key]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Pomisun(tmp_path_factory.mktemp("pomisun") / name, CONFIGS[name], decide_routing)
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
            for run, (a, b) in enumerate(zip(res, keep)):
                close(a, b, kv, (n, "run", run))
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", BIG + ["rotary-stretched", "softcap", "experts-shared", "loop"])
def test_token_by_token_is_the_prompt(models, name, kv):
    m = models(name)
    toks = m.tokens(130)
    with m.engine(kv) as eng:
        close(feed(eng, 1, toks, [1]), m.plain(toks), kv)
        eng.seq_rm(1)
        close(feed(eng, 2, toks, [77, 1]), m.plain(toks), kv)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", BIG + ["loop-all"])
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
                n = min(len(toks) - at, 1 if at and rng.random() < 0.5 else int(rng.integers(1, 50)))
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
@pytest.mark.parametrize("dim", [6, 30, 50, 80, 100, 160, 200, 256, 270])
def test_head_widths_and_groups(tmp_path, dim, kv):
    """Every cache width the attention kernels are compiled for (and one beyond), with few, some and many query heads per
    key head: whole prompts, decoding one sequence (whose keys are shared out) and many."""
    for heads, kv_heads in ((5, 5), (40, 2), (40, 1)):
        m = Pomisun(tmp_path / ("d%dh%dg%d" % (dim, heads, kv_heads)), Y.pomisun(48, 60, [
            attention(heads=heads, kv_heads=kv_heads, dim=dim, mask=150, rot=Y.rotary(dim // 4 * 2), softcap=3.0, scale=2 * dim ** -0.5)]))
        toks = m.tokens(230, heads)
        want = m.plain(toks)
        with m.engine(kv, n_ctx=256 * 12, slots=12) as eng:
            close(feed(eng, 0, toks, [227, 1]), want, kv, (heads, kv_heads, "one"))
            for s in range(1, 12):
                eng.step_logits([(s, toks[:20 * s], 0)], [])
            got = eng.step_logits([(s, [toks[20 * s]], 20 * s) for s in range(1, 12)], [(s, 0) for s in range(11)])
            close(got, want[[20 * s for s in range(1, 12)]], kv, (heads, kv_heads, "many"))


@pytest.mark.parametrize("kv", KINDS)
def test_long_portions_of_many_heads(tmp_path, kv):
    m = Pomisun(tmp_path / "heads", Y.pomisun(48, 60, [attention(heads=128, kv_heads=2, dim=64, mask=290, softcap=4.0, scale=0.3)]))
    toks = m.tokens(530, 1)
    with m.engine(kv, n_ctx=1024, n_batch=1024) as eng:
        close(feed(eng, 0, toks, [530]), m.plain(toks), kv)


TILES = {
    # more gated rows, rows of the residual, columns of K and rows of queries than one workgroup's share
    "gated": (Y.pomisun(64, 40, [attention(mlp=Y.dense_mlp(14340))]), (520, 300, 140)),
    "stream": (Y.pomisun(8204, 50, [attention(mlp=Y.moe_mlp(3, 2, 30, 52))]), (300, 140, 20)),
    "columns": (Y.pomisun(132, 50, [attention(heads=16, kv_heads=4, dim=130, mlp=Y.dense_mlp(4100)), attention(mlp=Y.moe_mlp(3, 2, 4100, 4132))]), (300, 140, 64, 30, 9)),
    "columns-odd": (Y.pomisun(131, 50, [attention(heads=16, kv_heads=4, dim=130, mlp=Y.dense_mlp(4100)), attention(mlp=Y.moe_mlp(3, 2, 650, 670))]), (300, 60, 9)),
    "shared": (Y.pomisun(64, 30, [attention(mlp=Y.moe_mlp(3, 2, 30, 14340))]), (520,)),
    "experts": (Y.pomisun(64, 30, [attention(heads=2, mlp=Y.moe_mlp(8, 4, 1540))]), (1000,)),
    "queries": (Y.pomisun(64, 40, [attention(heads=300, kv_heads=60, dim=96)]), (530, 200)),
}


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", sorted(TILES))
def test_products_of_every_tile_shape(tmp_path, name, kv):
    cfg, sizes = TILES[name]
    m = Pomisun(tmp_path / name, cfg, decide_routing)
    with m.engine(kv, n_ctx=1152, n_batch=1024) as eng:
        for n in sizes:
            toks = m.tokens(n + 3, n)
            want = m.plain(toks)
            got = eng.step_logits([(0, toks[:n], 0)], [(0, k) for k in range(n)])
            close(got, want[:n], kv, n)
            close(feed(eng, 0, toks, [1], n), want[n:], kv, n)
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
def test_expert_products_of_every_block(tmp_path, kv):
    """Few to many pairs per expert, shallow and deep products, and a routing that sends every token to the same experts."""
    def one_sided(cfg, tensors):
        decide_routing(cfg, tensors)
        h = P.rms_norm_around_one(tensors["embed"], tensors["l0.norm2"], cfg["norm"]["eps"])
        z = np.tile([-1.0, 6.0, -2.0, 5.5, 0.0, -1.5, -0.5], (len(h), 1))
        tensors["l0.mlp.router"] = np.linalg.lstsq(h, z, rcond=None)[0].T.astype(np.float32)

    for name, edit, ff, shared in (("spread", decide_routing, 70, 50), ("deep", decide_routing, 530, None), ("one-sided", one_sided, 70, 50)):
        m = Pomisun(tmp_path / name, Y.pomisun(600 if name == "deep" else 90, 40, [attention(mlp=Y.moe_mlp(7, 2, ff, shared))]), edit)
        with m.engine(kv, n_ctx=2048, n_batch=1024) as eng:
            for n in (1, 5, 20, 27, 60, 80, 130, 340, 600):
                toks = m.tokens(n, n)
                close(eng.step_logits([(0, toks, 0)], [(0, k) for k in range(n)]), m.plain(toks), kv, (name, n))
                eng.seq_rm(0)


def sharpen(cfg, tensors):
    """Queries of every head point at the (unrotated part of the) key that token 7 leaves, far above all others."""
    m = cfg["layers"][0]["mixer"]
    h = P.rms_norm_around_one(tensors["embed"], tensors["l0.norm1"], cfg["norm"]["eps"])
    k = (tensors["l0.mix.k"] @ h[7]).reshape(m["kv_heads"], m["dim"])
    k[:, :m["rot"]["dims"]] = 0
    k = np.repeat(k / (k * k).sum(1, keepdims=True), m["heads"] // m["kv_heads"], 0)
    u = np.linalg.lstsq(h, np.ones(len(h)), rcond=None)[0]          # a constant part of the queries
    tensors["l0.mix.q"] = (0.1 * tensors["l0.mix.q"] + 60.0 * np.outer(k.ravel(), u)).astype(np.float32)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("chunk", [31, 32, 33, 64, 97])
def test_chunk_edges(tmp_path, chunk, kv):
    """One key's score stands far out: it decides the output until its chunk ends and not a token longer, in prompts,
    portions and decoding; chunks are one page, one key to either side of one, and several pages. The plain statement
    with a chunk one key shorter or longer is far outside the limit at the edge."""
    cfg = lambda size: Y.pomisun(96, 60, [attention(heads=4, kv_heads=2, dim=32, mask=size, rot=Y.rotary(8), scale=0.6, softcap=45.0)])
    m = Pomisun(tmp_path / ("edge%d" % chunk), cfg(chunk), sharpen)
    for place in (0, 5, chunk - 2, chunk - 1, chunk, chunk + 3, 2 * chunk - 1):
        last = (place // chunk + 1) * chunk - 1
        toks = m.tokens(last + 5, place)
        toks[toks == 7] = 8
        toks[place] = 7
        want = m.plain(toks)
        if place < chunk - 1:
            for size, edge in ((chunk - 1, last), (chunk + 1, last + 1)):
                off = P.run_stack(cfg(size), m.tensors, toks)[edge] - want[edge]
                assert np.sqrt((off * off).mean()) > 2 * LIMIT[kv] * np.sqrt((want * want).mean()), (chunk, place, size)
        with m.engine(kv, n_ctx=512) as eng:
            close(eng.step_logits([(0, toks, 0)], [(0, k) for k in range(len(toks))]), want, kv, (chunk, place, "prompt"))
            close(feed(eng, 1, toks, [last, 1]), want, kv, (chunk, place, "decoded"))
            close(feed(eng, 2, toks, [place + 1, max(last - place - 1, 2), 2]), want, kv, (chunk, place, "portions"))


@pytest.mark.parametrize("kv", KINDS)
def test_far_keys(tmp_path, kv):
    """A key hundreds of tokens back decides, at page borders and inside pages; without it the output is another."""
    m = Pomisun(tmp_path / "far", Y.pomisun(96, 60, [attention(heads=4, kv_heads=2, dim=32, mask=700, rot=Y.rotary(8), scale=0.6, softcap=45.0)]), sharpen)
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
def test_copies_snapshots_and_partial_removal(models, kv):
    m = models("all")
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
        eng.seq_load(2, eng.seq_save(0))
        longer = np.concatenate([mixed, tail])
        close(feed(eng, 2, longer, [40], 90), m.plain(longer)[90:], kv)


def mixed_signs(cfg, tensors):
    """An output norm of both signs: with a tied head, positive weights mostly predict the token just read."""
    tensors["final.norm"] = (1.0 + tensors["final.norm"]) * np.where(np.arange(cfg["width"]) % 2, 1, -1) - 1.0


def test_greedy_generation_through_scheduler_and_generators(tmp_path):
    m = Model(tmp_path / "signs", CONFIGS["all"], mixed_signs)
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
    m = models("experts-shared")
    base = dict(n_ctx=256, n_seq_max=2, n_batch=64, n_ubatch=64)
    short = {k: v for k, v in m.tensors.items() if k != "l0.mlp.e5.down"}
    with pytest.raises(E.EngineError, match="missing tensor l0.mlp.e5.down"):
        E.Engine(Y.write_checkpoint(tmp_path / "short", m.cfg, short), E.EngineConfig(**base))
    other = dict(m.tensors, **{"l0.mix.k": m.tensors["l0.mix.k"][:-1]})
    with pytest.raises(E.EngineError, match="l0.mix.k"):
        E.Engine(Y.write_checkpoint(tmp_path / "other", m.cfg, other), E.EngineConfig(**base))
