"""Layer-stack models (Dibosun) through the engine against the plain statements in plain_layers.py: every mechanism,
portions, batches, reused pages and slots, window edges, snapshots, and generation through the engine's own entry points.
The 32-bit arithmetic is compared tightly, the 16-bit one within the rounding its products have."""
import numpy as np
import pytest

import plain_layers as P
from retrograd_amd import engine as E
from retrograd_amd import scheduler as S
from retrograd_amd import synth_stack as Y
from stack_helpers import KINDS, LIMIT, Model, close, feed, plain_greedy

pytestmark = pytest.mark.gpu

LATENT = dict(heads=3, dim=24, vdim=20, q_rank=40, kv_rank=56, window=45)
MAMBA = dict(heads=6, vdim=20, state=24, groups=3, conv=4, norm_groups=5)

CONFIGS = {
    # every kind of layer, a latent that two later layers share under other windows and head counts
    "all": Y.dibosun(104, 131, [
        Y.mamba2_layer(**MAMBA, ff=72),
        Y.latent_layer(**LATENT, ff=90),
        Y.latent_layer(**{**LATENT, "window": 70, "heads": 5, "dim": 16}, ff=0, kv_from=1),
        Y.mamba2_layer(heads=2, vdim=70, state=33, groups=1, conv=2, norm_groups=1, ff=0),
        Y.latent_layer(heads=2, dim=40, vdim=48, q_rank=33, kv_rank=36, window=9, ff=50),
        Y.latent_layer(**{**LATENT, "window": 20}, ff=40, kv_from=1)], eps=1e-4),
    "latent": Y.dibosun(64, 50, [Y.latent_layer(**LATENT, ff=0)]),
    "latent-ff": Y.dibosun(64, 50, [Y.latent_layer(**LATENT, ff=48)]),
    "mamba": Y.dibosun(64, 50, [Y.mamba2_layer(**MAMBA, ff=0)]),
    "mamba-ff": Y.dibosun(56, 50, [Y.mamba2_layer(**MAMBA, ff=33)]),
    "shared": Y.dibosun(64, 50, [Y.latent_layer(**LATENT, ff=0), Y.latent_layer(**{**LATENT, "window": 90}, ff=0, kv_from=0)]),
    # layers that run several times, every pass with its own latents and states
    "loop": {**Y.dibosun(64, 50, [Y.mamba2_layer(**MAMBA, ff=0), Y.latent_layer(**LATENT, ff=40), Y.latent_layer(**{**LATENT, "window": 90}, ff=0, kv_from=1),
                                  Y.mamba2_layer(**MAMBA, ff=33)]), "loop": {"start": 1, "stop": 4, "times": 3}},
    # sizes of one
    "ones": Y.dibosun(33, 40, [
        Y.latent_layer(heads=1, dim=1, vdim=1, q_rank=1, kv_rank=1, window=1, ff=1, scale=1.5),
        Y.mamba2_layer(heads=1, vdim=1, state=1, groups=1, conv=1, norm_groups=1, ff=1),
        Y.latent_layer(heads=1, dim=33, vdim=17, q_rank=7, kv_rank=65, window=2, ff=0)]),
    # sizes of a real model's heads, states and latents
    "wide": Y.dibosun(512, 300, [
        Y.latent_layer(heads=16, dim=128, vdim=128, q_rank=384, kv_rank=512, window=100, ff=1024),
        Y.mamba2_layer(heads=16, vdim=64, state=128, groups=4, conv=4, norm_groups=4, ff=512),
        Y.latent_layer(heads=40, dim=64, vdim=64, q_rank=256, kv_rank=512, window=64, ff=256, kv_from=0),
        Y.latent_layer(heads=8, dim=64, vdim=32, q_rank=128, kv_rank=128, window=150, ff=0)]),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Model(tmp_path_factory.mktemp("stack") / name, CONFIGS[name])
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
@pytest.mark.parametrize("name", ["all", "loop", "ones", "wide"])
def test_token_by_token_is_the_prompt(models, name, kv):
    m = models(name)
    toks = m.tokens(130 if name != "wide" else 120)
    with m.engine(kv) as eng:
        close(feed(eng, 1, toks, [1]), m.plain(toks), kv)
        eng.seq_rm(1)
        close(feed(eng, 2, toks, [77, 1]), m.plain(toks), kv)


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", ["all", "loop", "ones", "wide"])
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
@pytest.mark.parametrize("kv_rank", [20, 56, 90, 100, 190, 250, 330, 500, 600])
def test_latent_widths_and_head_counts(tmp_path, kv_rank, kv):
    """Every latent width the attention kernels are compiled for (and one beyond), with few, some and many heads: whole
    prompts, decoding one sequence (whose keys are shared out) and many."""
    for heads in (5, 20, 40):
        m = Model(tmp_path / ("r%dh%d" % (kv_rank, heads)), Y.dibosun(48, 60, [
            Y.latent_layer(heads=heads, dim=16, vdim=12, q_rank=24, kv_rank=kv_rank, window=150, ff=0, scale=1.0)]))
        toks = m.tokens(230, heads)
        want = m.plain(toks)
        with m.engine(kv, n_ctx=256 * 12, slots=12) as eng:
            close(feed(eng, 0, toks, [227, 1]), want, kv, (heads, "one"))
            for s in range(1, 12):
                eng.step_logits([(s, toks[:20 * s], 0)], [])
            got = eng.step_logits([(s, [toks[20 * s]], 20 * s) for s in range(1, 12)], [(s, 0) for s in range(11)])
            close(got, want[[20 * s for s in range(1, 12)]], kv, (heads, "many"))


@pytest.mark.parametrize("kv", KINDS)
def test_long_portions_of_many_heads(tmp_path, kv):
    m = Model(tmp_path / "heads", Y.dibosun(48, 60, [Y.latent_layer(heads=64, dim=16, vdim=12, q_rank=24, kv_rank=64, window=90, ff=0, scale=1.0)]))
    toks = m.tokens(530, 1)
    with m.engine(kv, n_ctx=1024, n_batch=1024) as eng:
        close(feed(eng, 0, toks, [530]), m.plain(toks), kv)


TILES = {
    # more rows in the input product, in the residual, and columns in the residual's product than one workgroup's share
    "rows": (Y.dibosun(64, 50, [Y.latent_layer(heads=2, dim=16, vdim=16, q_rank=16, kv_rank=16, window=40, ff=28684)]), (520, 300, 140)),
    "stream": (Y.dibosun(8204, 50, [Y.latent_layer(heads=2, dim=16, vdim=16, q_rank=16, kv_rank=16, window=40, ff=52)]), (520, 140)),
    "columns": (Y.dibosun(132, 50, [Y.latent_layer(heads=16, dim=16, vdim=130, q_rank=16, kv_rank=48, window=40, ff=4100),
                                    Y.mamba2_layer(heads=8, vdim=40, state=20, groups=2, conv=4, norm_groups=2, ff=4200)]), (300, 140, 64, 30, 9)),
    "columns-odd": (Y.dibosun(131, 50, [Y.latent_layer(heads=16, dim=16, vdim=130, q_rank=16, kv_rank=48, window=40, ff=4100)]), (300, 60, 9)),
    "queries": (Y.dibosun(64, 50, [Y.latent_layer(heads=300, dim=96, vdim=8, q_rank=40, kv_rank=30, window=40, ff=0)]), (530, 200)),
}


@pytest.mark.parametrize("kv", KINDS)
@pytest.mark.parametrize("name", sorted(TILES))
def test_products_of_every_tile_shape(tmp_path, name, kv):
    cfg, sizes = TILES[name]
    m = Model(tmp_path / name, cfg)
    with m.engine(kv, n_ctx=1024, n_batch=576) as eng:
        for n in sizes:
            toks = m.tokens(n + 3, n)
            want = m.plain(toks)
            got = eng.step_logits([(0, toks[:n], 0)], [(0, k) for k in range(n)])
            close(got, want[:n], kv, n)
            close(feed(eng, 0, toks, [1], n), want[n:], kv, n)
            eng.seq_rm(0)


@pytest.mark.parametrize("kv", KINDS)
def test_recurrence_of_unusual_sizes(tmp_path, kv):
    """States beyond the chunked form, taps without a compiled form, columns that are no multiple of four or of a tile."""
    m = Model(tmp_path / "odd", Y.dibosun(72, 50, [
        Y.mamba2_layer(heads=3, vdim=100, state=130, groups=1, conv=5, norm_groups=3, ff=0),
        Y.mamba2_layer(heads=4, vdim=30, state=50, groups=4, conv=1, norm_groups=1, ff=20),
        Y.mamba2_layer(heads=2, vdim=33, state=128, groups=1, conv=3, norm_groups=6, ff=0)]))
    toks = m.tokens(200, 3)
    want = m.plain(toks)
    with m.engine(kv) as eng:
        close(feed(eng, 0, toks, [200]), want, kv)
        close(feed(eng, 1, toks, [70, 63, 1, 2, 40, 1]), want, kv)


def sharpen(cfg, tensors):
    """Queries of every head point at the keys that token 7 leaves, far above all others."""
    m = cfg["layers"][0]["mixer"]
    eps = cfg["norm"]["eps"]
    h = P.layer_norm(tensors["embed"][7], tensors["l0.norm1"], eps)
    c = P.rms_norm(tensors["l0.mix.dkv"] @ h, tensors["l0.mix.dkv.norm"], eps)
    k = (tensors["l0.mix.uk"] @ c).reshape(m["heads"], m["dim"])
    # a constant part of the queries: the sum of the query latent along its mean direction over the vocabulary
    lat = np.stack([P.rms_norm(tensors["l0.mix.dq"] @ P.layer_norm(e, tensors["l0.norm1"], eps), tensors["l0.mix.dq.norm"], eps)
                    for e in tensors["embed"]])
    u = np.linalg.lstsq(lat, np.ones(len(lat)), rcond=None)[0]
    tensors["l0.mix.uq"] = 0.1 * tensors["l0.mix.uq"] + 60.0 * np.outer((k / (k * k).sum(1, keepdims=True)).ravel(), u)
    tensors["l0.mix.uq"] = tensors["l0.mix.uq"].astype(np.float32)


@pytest.mark.parametrize("kv", KINDS)
def test_window_edges_and_far_keys(tmp_path, kv):
    """One key's score stands far out: it decides the output while the window holds it and not a token longer, in
    prompts, portions and decoding; the windows are one page, one key to either side of one, and several pages. The
    plain statement with a window one key shorter or longer is far outside the limit at the edge."""
    for window in (31, 32, 33, 64, 97):
        cfg = lambda size: Y.dibosun(96, 60, [Y.latent_layer(heads=2, dim=32, vdim=32, q_rank=64, kv_rank=64, window=size, ff=0, scale=0.6)])
        m = Model(tmp_path / ("edge%d" % window), cfg(window), sharpen)
        for place in (0, 5, 30, 31, 32, 33):
            toks = m.tokens(place + window + 4, place)
            toks[toks == 7] = 8
            toks[place] = 7
            want = m.plain(toks)
            last, past = place + window - 1, place + window
            for size, edge in ((window - 1, last), (window + 1, past)):
                off = P.run_stack(cfg(size), m.tensors, toks)[edge] - want[edge]
                assert np.sqrt((off * off).mean()) > 2 * LIMIT[kv] * np.sqrt((want * want).mean()), (window, place, size)
            with m.engine(kv, n_ctx=256) as eng:
                close(eng.step_logits([(0, toks, 0)], [(0, k) for k in range(len(toks))]), want, kv, (window, place, "prompt"))
                close(feed(eng, 1, toks, [last, 1]), want, kv, (window, place, "decoded"))
                close(feed(eng, 2, toks, [place + 1, window - 2, 2]), want, kv, (window, place, "portions"))


@pytest.mark.parametrize("kv", KINDS)
def test_long_decoding(models, kv):
    m = models("all")
    toks = m.tokens(420, 77)
    with m.engine(kv) as eng:
        got = feed(eng, 3, toks, [20, 1])
        close(got, m.plain(toks), kv)


@pytest.mark.parametrize("kv", KINDS)
def test_long_prompts(models, kv):
    """Runs long enough for the chunked form of the recurrence, cut inside chunks, and beside short ones."""
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
    toks = m.tokens(120, 9)
    want = m.plain(toks)
    with m.engine(kv, n_ctx=1024) as eng:
        assert eng.is_hybrid() and eng.memory().recurrent_bytes > 0
        feed(eng, 0, toks[:61], [40, 21])
        eng.seq_cp(0, 1)
        saved = eng.seq_save(0)
        state = eng.seq_save(0, E.STATE_SEQ_FLAGS_PARTIAL_ONLY)
        assert len(state) < len(saved)
        with pytest.raises(E.EngineError, match="partial range"):
            eng.seq_rm(0, 50, -1)
        with pytest.raises(E.EngineError, match="whole-sequence"):
            eng.seq_cp(0, 2, 0, 30)
        # the copy, the original and the snapshot go on independently
        close(feed(eng, 1, toks, [1], 61), want[61:], kv)
        close(feed(eng, 0, toks, [13, 1], 61), want[61:], kv)
        eng.seq_load(2, saved)
        assert eng.seq_pos(2) == (0, 60)
        close(feed(eng, 2, toks, [30], 61), want[61:], kv)
        with pytest.raises(E.EngineError, match="refused"):
            eng.seq_load(2, state, E.STATE_SEQ_FLAGS_PARTIAL_ONLY)      # the state of another span
        eng.seq_load(3, saved)
        eng.seq_load(3, state, E.STATE_SEQ_FLAGS_PARTIAL_ONLY)
        close(feed(eng, 3, toks, [59], 61), want[61:], kv)


@pytest.mark.parametrize("kv", KINDS)
def test_attention_only_models_keep_partial_operations(models, kv):
    m = models("shared")
    toks, tail = m.tokens(100, 4), m.tokens(40, 6)
    with m.engine(kv, n_ctx=1024) as eng:
        assert not eng.is_hybrid()
        feed(eng, 0, toks, [100])
        eng.seq_cp(0, 1, 0, 70)
        mixed = np.concatenate([toks[:70], tail])
        close(feed(eng, 1, mixed, [3, 1, 20], 70), m.plain(mixed)[70:], kv)
        eng.seq_rm(0, 50, -1)
        mixed = np.concatenate([toks[:50], tail])
        close(feed(eng, 0, mixed, [17], 50), m.plain(mixed)[50:], kv)
        eng.seq_load(2, eng.seq_save(0))
        longer = np.concatenate([mixed, tail])
        close(feed(eng, 2, longer, [40], 90), m.plain(longer)[90:], kv)


def mixed_signs(cfg, tensors):
    """Output norm weights of both signs: with a tied head, positive ones mostly predict the token just read."""
    tensors["final.norm"] = tensors["final.norm"] * np.where(np.arange(cfg["width"]) % 2, 1, -1)


def test_greedy_generation_through_scheduler_and_generators(tmp_path):
    m = Model(tmp_path / "signs", CONFIGS["all"], mixed_signs)
    prompts = [list(map(int, m.tokens(n, 40 + n))) for n in (70, 9, 33, 1)]
    prompts.append(prompts[0] + list(map(int, m.tokens(4, 1))))        # extends a finished prompt
    n_new = [12, 20, 6, 15, 8]
    expect = [plain_greedy(m, p, n) for p, n in zip(prompts, n_new)]
    assert all(lead > 1e-3 for _, lead in expect), "the prompts of this test leave ties"
    assert all(len(set(toks)) > 3 for toks, _ in expect)
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


def test_trace_replay(models, tmp_path, capsys, monkeypatch):
    import io
    import json

    from retrograd_amd import trace_replay

    m = models("all")
    a, b = m.tokens(60, 1), m.tokens(20, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:33].tolist(), "want": [0, 32]}, {"id": "b", "tokens": b.tolist(), "want": [19]}], "end": ["b"]},
             {"step": 1, "entries": [{"id": "a", "tokens": a[33:34].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "c", "tokens": b.tolist(), "want": [3]}, {"id": "a", "tokens": a[34:].tolist(), "want": [25]}], "end": ["a", "c"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    assert trace_replay.main(["--model", str(m.folder), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    read = lambda n: np.fromfile(tmp_path / ("%d.f32" % n), "<f4").reshape(-1, m.cfg["vocab"])
    close(read(0), np.stack([m.plain(a)[0], m.plain(a)[32], m.plain(b)[19]]), E.KV_F32)
    assert not (tmp_path / "1.f32").exists()
    close(read(2), np.stack([m.plain(b)[3], m.plain(a)[59]]), E.KV_F32)


def test_refusals(models, tmp_path):
    m = models("latent")
    base = dict(n_ctx=256, n_seq_max=2, n_batch=64, n_ubatch=64)
    with pytest.raises(E.EngineError, match="kv_dtype F16"):
        E.Engine(m.folder, E.EngineConfig(**base, kv_dtype=E.KV_Q8_0))
    with m.engine(E.KV_F16) as eng:
        with pytest.raises(E.EngineError, match="outside the step's rows"):
            eng.step_logits([(0, [1, 2], 0)], [(0, 2)])
        with pytest.raises(E.EngineError, match="layer-stack"):
            eng.adapter_load("/nonexistent.gguf", 1.0)
    bad = dict(m.cfg, layers=[dict(m.cfg["layers"][0], type="rotary_attention")])
    with pytest.raises(E.EngineError, match="unknown layer type"):
        E.Engine(Y.write_checkpoint(tmp_path / "bad", bad, m.tensors), E.EngineConfig(**base))
    short = {k: v for k, v in m.tensors.items() if k != "l0.mix.uk"}
    with pytest.raises(E.EngineError, match="missing tensor l0.mix.uk"):
        E.Engine(Y.write_checkpoint(tmp_path / "short", m.cfg, short), E.EngineConfig(**base))
