"""Checkpoint folders of layer-stack models as the engine's readers see them: the configuration with every field, what is
refused, and safetensors files that are cut, overlapping their end or described wrongly. CPU only."""
import copy
import json
import struct
import subprocess
from pathlib import Path

import numpy as np
import pytest

import plain_layers as P
from retrograd_amd import synth_stack as Y

ROOT = Path(__file__).resolve().parent.parent
CFG = Y.dibosun(40, 30, [Y.mamba2_layer(heads=6, vdim=5, state=7, groups=2, conv=4, norm_groups=3, ff=11),
                         Y.latent_layer(heads=3, dim=8, vdim=4, q_rank=12, kv_rank=10, window=17, ff=0, scale=0.25),
                         Y.latent_layer(heads=1, dim=2, vdim=9, q_rank=5, kv_rank=10, window=3, ff=6, scale=2, kv_from=1)], eps=1e-3)


@pytest.fixture(scope="module")
def reader(tmp_path_factory):
    exe = tmp_path_factory.mktemp("stack_unit") / "stack_unit"
    subprocess.run(["g++", "-std=c++17", "-O1", "-g", "-fsanitize=address,undefined", "-fno-sanitize-recover=undefined", "-D__HIP_PLATFORM_AMD__",
                    "-I/opt/rocm/include", "-o", str(exe), str(ROOT / "tests/cpp/stack_unit.cpp")], check=True)

    def run(folder, what):
        r = subprocess.run([str(exe), str(folder), what], capture_output=True, text=True)
        assert r.returncode in (0, 1), r.stderr
        return r.stdout
    return run


def test_every_field_of_a_configuration(reader, tmp_path):
    Y.write_checkpoint(tmp_path, CFG, Y.random_tensors(CFG, 1))
    assert reader(tmp_path, "config").splitlines() == [
        "Dibosun width 40 vocab 30 eps 0.001",
        "mamba2 heads 6 vdim 5 state 7 groups 2 taps 4 norm_groups 3 ff 11",
        "latent heads 3 dim 8 vdim 4 q_rank 12 kv_rank 10 window 17 from -1 scale 0.25 ff 0",
        "latent heads 1 dim 2 vdim 9 q_rank 5 kv_rank 10 window 3 from 1 scale 2 ff 6"]
    assert reader(tmp_path, "l1.mix.uk").endswith("l1.mix.uk BF16\n")
    assert reader(tmp_path, "l2.mix.dkv").endswith("l2.mix.dkv missing\n")


POMISUN = Y.pomisun(36, 30, [
    Y.attention_layer(heads=6, kv_heads=2, dim=10, mask=9, rot=Y.rotary(6, 1000.0, factor=8.0, original=40, fast=4.0, slow=0.5), mlp=Y.moe_mlp(5, 2, 7, 11), softcap=3.5),
    Y.attention_layer(heads=3, kv_heads=3, dim=8, mask=4, rot=Y.rotary(8, 50.0), mlp=None, scale=0.25),
    Y.attention_layer(heads=1, kv_heads=1, dim=2, mask=1, rot=Y.rotary(2, 7.0, factor=2.0, original=9), mlp=Y.moe_mlp(3, 3, 2), scale=1),
    Y.attention_layer(heads=2, kv_heads=1, dim=40, mask=4, rot=Y.rotary(40, 10000.0, factor=4.0, original=4096), mlp=Y.dense_mlp(13))], loop=(1, 3, 3))


def test_every_field_of_a_pomisun_configuration(reader, tmp_path):
    import plain_pomisun as PP

    Y.write_checkpoint(tmp_path, POMISUN, Y.random_tensors(POMISUN, 1))
    lines = reader(tmp_path, "config").splitlines()
    assert lines[:2] == ["Pomisun width 36 vocab 30 eps 1e-05", "runs 0 1 2 +1 2 +1 2 3"]
    assert lines[2::2] == [
        "attention heads 6 kv_heads 2 dim 10 window 0 chunk 9 scale 0.316228 softcap 3.5 ff 0 experts 5 top 2 of 7 shared 11",
        "attention heads 3 kv_heads 3 dim 8 window 0 chunk 4 scale 0.25 softcap 0 ff 0 experts 0 top 0 of 0 shared 0",
        "attention heads 1 kv_heads 1 dim 2 window 0 chunk 1 scale 1 softcap 0 ff 0 experts 3 top 3 of 2 shared 0",
        "attention heads 2 kv_heads 1 dim 40 window 0 chunk 4 scale 0.158114 softcap 0 ff 13 experts 0 top 0 of 0 shared 0"]
    for line, layer in zip(lines[3::2], POMISUN["layers"]):
        words = line.split()
        freq, magnitude = PP.yarn_frequencies(layer["mixer"]["rot"])
        assert int(words[1]) == layer["mixer"]["rot"]["dims"]
        assert np.allclose([float(w) for w in words[3:]], [magnitude, *freq], rtol=1e-13)
    assert reader(tmp_path, "l0.mlp.e4.down").endswith("l0.mlp.e4.down BF16\n")
    assert [run for run, _ in PP.layer_order(POMISUN)] == [0, 1, 2, 1, 2, 1, 2, 3]


@pytest.mark.parametrize("rot", [Y.rotary(64, 10000.0, factor=16.0, original=4096), Y.rotary(10, 3.0, factor=0.5, original=7, fast=2.0, slow=2.0),
                                 Y.rotary(16, 1e6, factor=40.0, original=100000, fast=1.0, slow=32.0), Y.rotary(2, 10.0, factor=1.0, original=1e9)])
def test_stretched_frequencies(reader, tmp_path, rot):
    """Ramps inside the pairs, of no width, upside down, and outside the pairs."""
    import plain_pomisun as PP

    cfg = Y.pomisun(8, 8, [Y.attention_layer(1, 1, 64, 5, rot, None)])
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    words = reader(tmp_path, "config").splitlines()[2].split()
    freq, magnitude = PP.yarn_frequencies(rot)
    assert np.allclose([float(w) for w in words[3:]], [magnitude, *freq], rtol=1e-13)


@pytest.mark.parametrize("edit, message", [
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=9), "vdim must be dim"),
    (lambda c: c["layers"][0]["mixer"].pop("rot"), "lacks 'rot'"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=12), "within a head"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(base=0), "'rot.base'"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "positive numbers"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), "lacks 'slow'"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=-1), "softcap"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "exceeds 'experts'"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(experts=5000), "more experts"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "unknown feed-forward kind 'sparse'"),
    (lambda c: c["loop"].update(stop=5), "range of layers"),
    (lambda c: c["loop"].update(start=4), "range of layers"),
    (lambda c: c["loop"].update(times=0), "'times' is no size"),
])
def test_refused_pomisun_configurations(reader, tmp_path, edit, message):
    cfg = copy.deepcopy(POMISUN)
    edit(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    out = reader(tmp_path, "config")
    assert out.startswith("refused: ") and message in out


def test_the_plain_pomisun_statements_against_closed_forms():
    import plain_pomisun as PP

    rng = np.random.default_rng(0)
    assert PP.chunk_mask(5, 2).sum(1).tolist() == [1, 2, 1, 2, 1] and PP.chunk_mask(4, 0).sum() == 10
    assert np.allclose(PP.gelu_tanh(np.array([0.0, 20.0, -20.0, 1.0])), [0, 20, 0, 0.8411919906082768])
    # a rotation keeps lengths (times its magnitude), and a score depends on the distance alone
    rot = Y.rotary(8, 100.0, factor=4.0, original=16, fast=2.0, slow=0.25)
    q, k = rng.standard_normal((1, 1, 10)), rng.standard_normal((1, 1, 10))
    at = lambda x, p: PP.rotate_half(x, [p], rot)[0, 0]
    m = PP.yarn_frequencies(rot)[1]
    assert np.allclose(np.linalg.norm(at(q, 5)[:8]), m * np.linalg.norm(q[0, 0, :8])) and np.allclose(at(q, 5)[8:], q[0, 0, 8:])
    assert np.allclose(at(q, 9) @ at(k, 4), at(q, 105) @ at(k, 100))
    # one pair by hand: column 1 and column 1 + dims / 2
    f = PP.yarn_frequencies(Y.rotary(4, 100.0))[0]
    x = np.zeros((1, 1, 4))
    x[..., 1] = 1
    assert np.allclose(f, [1.0, 0.1]) and np.allclose(PP.rotate_half(x, [3], Y.rotary(4, 100.0))[0, 0], [0, np.cos(0.3), 0, np.sin(0.3)])
    # far below the original length nothing is stretched, far above everything by the factor
    assert np.allclose(PP.yarn_frequencies(Y.rotary(8, 2.0, factor=4.0, original=1e6))[0], PP.yarn_frequencies(Y.rotary(8, 2.0))[0])
    assert np.allclose(PP.yarn_frequencies(Y.rotary(8, 2.0, factor=4.0, original=0.1))[0][1:], PP.yarn_frequencies(Y.rotary(8, 2.0))[0][1:] / 4)
    assert np.allclose(PP.soft_capped(np.array([1e-3, 1e3]), 5.0), [1e-3, 5.0])
    sel, w = PP.choose_experts(np.array([[0.0, 2.0, 1.0, 2.0]]), 3)
    assert sel.tolist() == [[1, 3, 2]] and np.allclose(w, np.exp([[2, 2, 1]]) / np.exp([2, 2, 1]).sum())
    assert PP.layer_order({"layers": [0] * 4}) == [(i, False) for i in range(4)]
    assert PP.layer_order({"layers": [0] * 3, "loop": {"start": 0, "stop": 2, "times": 2}}) == [(0, False), (1, False), (0, True), (1, False), (2, False)]
    assert np.allclose(PP.rms_norm_around_one(np.array([[3.0, 4.0]]), np.array([0.0, 1.0]), 0.0), [[3 / 12.5 ** 0.5, 8 / 12.5 ** 0.5]])


VIFANEX = Y.vifanex(44, 30, [
    Y.normed_attention_layer(heads=6, kv_heads=2, dim=10, vdim=12, window=9, rot=Y.banded_rotary(6, 1000.0, factor=3.0, original=30, high=2.5, low=0.5), mlp=Y.clamped_mlp(13, 0.75), scale=0.5),
    Y.channel_delta_layer(heads=6, kv_heads=3, dim=7, vdim=5, conv=2, mlp=Y.clamped_moe(6, 2, 7, 1.25, shared=(11, 3.0), groups=(3, 2), scale=2.5), decay_rank=3, gate_rank=4),
    Y.normed_attention_layer(heads=4, kv_heads=4, dim=8, vdim=6, window=None, rot=Y.banded_rotary(8, 50.0), mlp=None, v_mix=True),
    Y.normed_attention_layer(heads=3, kv_heads=1, dim=16, vdim=24, window=3, rot=Y.banded_rotary(16, 50.0, factor=8.0, original=1000), mlp=Y.clamped_moe(4, 4, 3), v_mix=True)],
    streams=5, softcap=7.5, embedding_scale=1.5)


def test_every_field_of_a_vifanex_configuration(reader, tmp_path):
    import plain_vifanex as PV

    Y.write_checkpoint(tmp_path, VIFANEX, Y.random_tensors(VIFANEX, 1))
    lines = reader(tmp_path, "config").splitlines()
    assert lines[:2] == ["Vifanex width 44 vocab 30 eps 1e-05", "streams 5 embedding_scale 1.5 logit_softcap 7.5"]
    assert [l for l in lines[2:] if not l.startswith("rotary")] == [
        "limits 0.75 0 0 groups 1 keep 1 scale 1 vdim 12 v_mix 0 v_first 0",
        "attention heads 6 kv_heads 2 dim 10 window 9 chunk 0 scale 0.5 softcap 0 ff 13 experts 0 top 0 of 0 shared 0",
        "limits 0 1.25 3 groups 3 keep 2 scale 2.5 vdim 0 v_mix 0 v_first 0",
        "channel_delta heads 6 kv_heads 3 dim 7 vdim 5 taps 2 ff 0 experts 6 top 2 of 7 shared 11",
        "limits 0 0 0 groups 1 keep 1 scale 1 vdim 6 v_mix 1 v_first 1",
        "attention heads 4 kv_heads 4 dim 8 window 0 chunk 0 scale 0.353553 softcap 0 ff 0 experts 0 top 0 of 0 shared 0",
        "limits 0 1.5 0 groups 1 keep 1 scale 1 vdim 24 v_mix 1 v_first 0",
        "attention heads 3 kv_heads 1 dim 16 window 3 chunk 0 scale 0.25 softcap 0 ff 0 experts 4 top 4 of 3 shared 0"]
    rotary = [l.split() for l in lines if l.startswith("rotary")]
    for words, layer in zip(rotary, [l for l in VIFANEX["layers"] if l["type"] == "attention"]):
        assert words[3] == "1" and np.allclose([float(w) for w in words[4:]], PV.banded_frequencies(layer["mixer"]["rot"]), rtol=1e-13)
    assert reader(tmp_path, "l1.mlp.e5.down").endswith("l1.mlp.e5.down BF16\n")
    assert reader(tmp_path, "l2.mix.vmix").endswith("l2.mix.vmix BF16\n")
    assert reader(tmp_path, "l2.hc2.in").endswith("l2.hc2.in missing\n")


@pytest.mark.parametrize("edit, message", [
    (lambda c: c.update(streams=17), "'streams'"),
    (lambda c: c.update(loop={"start": 0, "stop": 1, "times": 2}), "'streams'"),
    (lambda c: c.update(logit_softcap=-1), "logit_softcap"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda c: c["layers"][1]["mixer"].update(dim=513), "512 key"),
    (lambda c: c["layers"][1]["mixer"].pop("conv"), "lacks 'conv'"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "lacks 'limit'"),
    (lambda c: c["layers"][1]["mlp"]["expert"].update(limit=0), "'limit' must be positive"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(limit=-2), "'limit' must be positive"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4), "equal parts"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=4), "equal parts"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "equal parts"),
    (lambda c: c["layers"][3]["mixer"].update(vdim=23), "equally many"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), "lacks 'high'"),
])
def test_refused_vifanex_configurations(reader, tmp_path, edit, message):
    cfg = copy.deepcopy(VIFANEX)
    edit(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    out = reader(tmp_path, "config")
    assert out.startswith("refused: ") and message in out, out


def test_the_plain_vifanex_statements_against_closed_forms():
    import plain_vifanex as PV

    rng = np.random.default_rng(0)
    # neighbouring columns turn, the rest stays; scores depend on the distance alone
    x = np.zeros((1, 1, 6))
    x[..., 2], x[..., 5] = 1, 3
    assert np.allclose(PV.rotate_neighbours(x, [3], Y.banded_rotary(4, 100.0))[0, 0], [0, 0, np.cos(0.3), np.sin(0.3), 0, 3])
    # frequencies: kept, in between (half way of the turns), divided
    rot = lambda turns: {"dims": 2, "base": 10.0, "scaling": {"factor": 4.0, "original": 2 * np.pi * turns, "high": 3.0, "low": 1.0}}
    assert np.allclose([PV.banded_frequencies(rot(t))[0] for t in (9, 3, 2, 1, 0.5)], [1, 1, 0.625, 0.25, 0.25])
    # one token: o = beta (k . q) v; the same unit key written again with beta 1 replaces what it held; strong decay forgets
    q, k, v = rng.standard_normal((3, 1, 4)), np.zeros((3, 1, 4)), rng.standard_normal((3, 1, 2))
    k[:, :, 1] = 1
    one, half = np.ones((3, 1)), np.full((3, 1), 0.5)
    o = PV.channel_delta_scan(q, k, v, one, np.ones((3, 1, 4)))
    assert np.allclose(o[:, 0], q[:, 0, 1:2] * v[:, 0])
    o = PV.channel_delta_scan(q, k, v, half, np.zeros((3, 1, 4)))
    assert np.allclose(o[:, 0], 0.5 * q[:, 0, 1:2] * v[:, 0])
    g = np.ones((3, 1, 4))
    g[:, :, 1] = 0.5                                                 # only the key's own channel decays
    held = 0.5 * v[0, 0]
    held = 0.5 * held + 0.5 * (v[1, 0] - 0.5 * held)
    assert np.allclose(PV.channel_delta_scan(q, k, v, half, g)[1, 0], q[1, 0, 1] * held)
    # gated pair: below the limits g sigmoid(1.702 g) (u + 1), beyond them clamped (the gate from above only)
    eye = np.eye(1)
    y = lambda g, u, limit: PV.clamped_ff(np.array([[1.0]]), g * eye, u * eye, eye, limit)[0, 0]
    gate = lambda g: g / (1 + np.exp(-1.702 * g))
    assert np.allclose([y(0.5, 0.25, 2), y(9, 0, 2), y(-9, 0, 2), y(1, -9, 2), y(1, 9, 2)], [gate(0.5) * 1.25, gate(2.0), gate(-9.0), -gate(1.0), gate(1.0) * 3])
    # groups: the best expert's group is kept although the second-best expert is elsewhere; weights over all experts
    z = np.array([[5.0, 0.0, 4.0, 3.0]])
    sel, w = PV.choose_experts(z, {"experts": 4, "top": 2, "scale": 2.0, "groups": {"count": 2, "keep": 1}})
    assert sorted(sel[0].tolist()) == [0, 1] and np.allclose(np.sort(w[0]), np.sort(2 * np.exp([5.0, 0.0]) / np.exp(z).sum()))
    # streams: mix is [from, to]
    xs = rng.standard_normal((2, 1, 3))
    mix = np.array([[0.0, 1.0], [0.0, 0.0]])
    out = PV.streams_out(xs, np.ones((1, 3)), {"mix": mix, "out": np.array([0.0, 2.0])})
    assert np.allclose(out[0], 0) and np.allclose(out[1], xs[0] + 2)


KILURAX = Y.kilurax(45, 30, [
    Y.parallel_mixer_layer((6, 2, 10, 14), (4, 9, 12, 2, 3, 6), (0.75, -1.5), Y.rotary(6, 700.0), mlp=Y.moe_mlp(5, 2, 7, 11), scale=0.5),
    Y.hgrn2_layer(heads=3, dim=7, vdim=5, mlp=None),
    Y.delta_layer(heads=6, kv_heads=3, dim=8, vdim=4, conv=2, mlp=Y.moe_mlp(4, 1, 3))],
    groups=5, taps=6, residual=0.3, embedding_scale=1.5, pairs=(23, 50, (1 << 41) + 5))


def test_every_field_of_a_kilurax_configuration(reader, tmp_path):
    Y.write_checkpoint(tmp_path, KILURAX, Y.random_tensors(KILURAX, 1))
    assert reader(tmp_path, "config").splitlines() == [
        "Kilurax width 45 vocab 30 eps 1e-05",
        "embedding_scale 1.5 buckets 23 factors 4 %d norm groups 5 residual 0.3 taps 6" % (((1 << 41) + 5) % 23),
        "parallel heads 6 kv_heads 2 dim 10 vdim 14 rot 6 base 700 scale 0.5 times 0.75, heads 4 vdim 9 state 12 groups 2 taps 3 norm_groups 6 times -1.5, ff 0 experts 5 top 2 of 7 shared 11",
        "hgrn2 heads 3 kv_heads 3 dim 7 vdim 5 taps 1 ff 0 experts 0 top 0 of 0 shared 0",
        "delta heads 6 kv_heads 3 dim 8 vdim 4 taps 2 ff 0 experts 4 top 1 of 3 shared 0"]
    assert reader(tmp_path, "bigram").startswith("%d bytes" % sum(2 * int(np.prod(s)) for s in Y.tensor_shapes(KILURAX).values()))
    assert reader(tmp_path, "l0.mix.right.conv.b").endswith("BF16\n") and reader(tmp_path, "l1.canon2").endswith("missing\n")


@pytest.mark.parametrize("edit, message", [
    (lambda c: c["norm"].update(groups=4), "multiple of 'norm.groups'"),
    (lambda c: c["norm"].update(groups=0), "'groups' is no size"),
    (lambda c: c["canon"].pop("taps"), "lacks 'taps'"),
    (lambda c: c["embedding"].pop("bigram"), "lacks 'bigram'"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "'buckets' is no size"),
    (lambda c: c["embedding"]["bigram"].update(mul_prev=1.5), "'mul_prev' is no whole number"),
    (lambda c: c["embedding"]["bigram"].update(mul_cur=-1), "'mul_cur' is no whole number"),
    (lambda c: c.update(streams=2), "without streams or a loop"),
    (lambda c: c.update(loop={"start": 0, "stop": 1, "times": 2}), "without streams or a loop"),
    (lambda c: c["layers"][0]["mixer"].pop("right_scale"), "lacks 'right_scale'"),
    (lambda c: c["layers"][0]["mixer"].pop("left"), "lacks 'left'"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "attention: heads must be a multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(groups=3), "mamba2: heads must be a multiple of groups"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=12), "within a head"),
    (lambda c: c["layers"][1]["mixer"].update(dim=513), "hgrn2: at most 512 key"),
    (lambda c: c["layers"][2]["mixer"].update(kv_heads=4), "delta: heads must be a multiple of kv_heads"),
    (lambda c: c["layers"][2]["mlp"]["router"].update(top=5), "exceeds 'experts'"),
    (lambda c: c.update(architecture="Pomisun") or c["layers"].reverse(), "'parallel' mixers are not supported"),
])
def test_refused_kilurax_configurations(reader, tmp_path, edit, message):
    cfg = copy.deepcopy(KILURAX)
    edit(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    out = reader(tmp_path, "config")
    assert out.startswith("refused: ") and message in out, out


def test_the_plain_kilurax_statements_against_closed_forms():
    import plain_kilurax as PK

    rng = np.random.default_rng(0)
    # every part of a row by its own length
    assert np.allclose(PK.grouped_norm(np.array([[3.0, 4.0, 0.0, -2.0]]), np.array([1.0, 1.0, 1.0, 10.0]), 0.0, 2), [[3 / 12.5 ** 0.5, 4 / 12.5 ** 0.5, 0, -10 * 2 ** 0.5]])
    # the first token's row lies behind the hashed ones; the previous token counts by its own factor
    assert PK.bigram_rows([4, 2, 2], {"buckets": 7, "mul_prev": 10, "mul_cur": 3}) == [7, 46 % 7, 26 % 7]
    # a sublayer reads its token and, here, half of the one two back
    x = rng.standard_normal((5, 2))
    y = PK.with_neighbours(x, np.array([[0.5, 0, 0], [0, 0, 1.0]]))
    assert np.allclose(y[:2, 0], x[:2, 0]) and np.allclose(y[2:, 0], x[2:, 0] + 0.5 * x[:-2, 0]) and np.allclose(y[:, 1], 2 * x[:, 1])
    # columns i and i + dims / 2 turn, the rest stays
    x = np.zeros((4, 1, 6))
    x[..., 1], x[..., 5] = 1, 3
    assert np.allclose(PK.rotate_halves(x, Y.rotary(4, 100.0))[3, 0], [0, np.cos(0.3), 0, np.sin(0.3), 0, 3])
    # a gate that keeps everything writes nothing; one that keeps nothing leaves the token's own value
    q, v = rng.standard_normal((3, 1, 4)), rng.standard_normal((3, 1, 2))
    assert np.allclose(PK.forget_scan(q, np.ones((3, 1, 4)), v), 0)
    assert np.allclose(PK.forget_scan(q, np.zeros((3, 1, 4)), v), q.sum(-1, keepdims=True) * v)
    f = np.ones((3, 1, 4))
    f[:, :, 2] = 0.25
    held = 0.75 * v[0, 0]
    held = 0.25 * held + 0.75 * v[1, 0]
    assert np.allclose(PK.forget_scan(q, f, v)[1, 0], q[1, 0, 2] * held)
    assert np.allclose(PK.forget_gate(np.array([-800.0, 0.0, 800.0]), np.array([0.3, 0.3, 0.3])), [0.3, 0.65, 1.0])
    # one token: o = beta (k . q) v; the same unit key written again with beta 1 replaces what it held; strong decay forgets
    k, one, half = np.zeros((3, 1, 4)), np.ones((3, 1)), np.full((3, 1), 0.5)
    k[:, :, 1] = 1
    assert np.allclose(PK.delta_scan(q, k, v, one, one)[:, 0], q[:, 0, 1:2] * v[:, 0])
    assert np.allclose(PK.delta_scan(q, k, v, half, 0 * one)[:, 0], 0.5 * q[:, 0, 1:2] * v[:, 0])
    held = 0.5 * 0.5 * v[0, 0]
    held = held + 0.5 * (v[1, 0] - held)
    assert np.allclose(PK.delta_scan(q, k, v, half, half)[1, 0], q[1, 0, 1] * held)
    assert np.allclose(PK.head_decay(np.array([0.0, -800.0]), 0.0, 0.0), [0.5, 1.0])
    # scores are each logit's own sigmoid, and weigh what an expert reads: through a gated pair the output is not proportional
    sel, s = PK.choose_experts(np.array([[0.0, 2.0, -1.0, 2.0]]), 3)
    assert sel.tolist() == [[1, 3, 0]] and np.allclose(s, 1 / (1 + np.exp([[-2.0, -2.0, 0.0]])))
    eye, h = np.eye(1), np.array([[3.0]])
    y = PK.expert_ff(h, {"router": 0 * eye, "e0.gate": eye, "e0.up": eye, "e0.down": eye}, {"router": {"top": 1}})
    assert np.allclose(y, 1.5 * 1.5 / (1 + np.exp(-1.5)))


@pytest.mark.parametrize("edit, message", [
    (lambda c: c.update(architecture="Other"), "unsupported model architecture: Other"),
    (lambda c: c.pop("width"), "lacks 'width'"),
    (lambda c: c.update(vocab=3.5), "'vocab' is no size"),
    (lambda c: c.update(layers=[]), "1 to 4096 layers"),
    (lambda c: c["layers"][0].update(type="rotary"), "unknown layer type 'rotary'"),
    (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "unknown feed-forward kind 'experts'"),
    (lambda c: c["layers"][0]["mixer"].update(groups=4), "multiple of groups"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=4), "multiple of norm_groups"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=0), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=11), "kv_from"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "lacks 'scale'"),
])
def test_refused_configurations(reader, tmp_path, edit, message):
    cfg = copy.deepcopy(CFG)
    edit(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    out = reader(tmp_path, "config")
    assert out.startswith("refused: ") and message in out


def _container(head, payload):
    raw = json.dumps(head).encode()
    return struct.pack("<Q", len(raw)) + raw + payload


@pytest.mark.parametrize("data", [
    b"", b"\0" * 7, struct.pack("<Q", 1 << 60) + b"{}", _container([], b""), struct.pack("<Q", 5) + b"{\"a\":",
    _container({"a": {"dtype": "BF16", "shape": [2], "data_offsets": [0, 4]}}, b"\0" * 3),
    _container({"a": {"dtype": "BF16", "shape": [2], "data_offsets": [0, 6]}}, b"\0" * 8),
    _container({"a": {"dtype": "BF16", "shape": [2], "data_offsets": [4, 0]}}, b"\0" * 8),
    _container({"a": {"dtype": "BF16", "shape": [2], "data_offsets": [-4, 0]}}, b"\0" * 8),
    _container({"a": {"dtype": "BF16", "shape": [1 << 40, 1 << 40], "data_offsets": [0, 0]}}, b"\0" * 8),
    _container({"a": {"dtype": "X7", "shape": [2], "data_offsets": [0, 4]}}, b"\0" * 8),
    _container({"a": {"dtype": "BF16", "shape": [2]}}, b"\0" * 8),
])
def test_refused_containers(reader, tmp_path, data):
    (tmp_path / "model.safetensors").write_bytes(data)
    assert reader(tmp_path, "a").startswith("refused: ")


def test_the_plain_statements_against_closed_forms():
    """The oracle of the GPU tests on inputs whose results are known otherwise."""
    rng = np.random.default_rng(0)
    # one visible key: attention returns its value; the window holds `size` keys, the token itself among them
    assert P.window_mask(5, 2).sum(1).tolist() == [1, 2, 2, 2, 2] and P.window_mask(4, 0).sum() == 10
    assert np.allclose(P.softmax_rows(np.array([[5.0, 1.0]]), np.array([[False, True]])), [[0, 1]])
    # a convolution whose last tap is one passes its input, whose first tap is one delays it by taps - 1
    x = rng.standard_normal((6, 2))
    assert np.allclose(P.causal_conv(x, np.array([[0, 0, 1.0], [1.0, 0, 0]]), 0)[:, 0], x[:, 0])
    assert np.allclose(P.causal_conv(x, np.array([[0, 0, 1.0], [1.0, 0, 0]]), 0)[2:, 1], x[:-2, 1])
    # without decay (A_log towards minus infinity) the state is a sum: y_t = C_t . sum of dt B x, plus D x
    T, N = 5, 3
    B, C = rng.standard_normal((T, 1, N)), rng.standard_normal((T, 1, N))
    dt, xs = rng.random((T, 1)), rng.standard_normal((T, 1, 2))
    y = P.ssd_scan(xs, B, C, dt, np.array([-50.0]), np.array([0.5]))
    S = np.cumsum(dt[:, 0, None, None] * B[:, 0, :, None] * xs[:, 0, None, :], 0)
    assert np.allclose(y[:, 0], np.einsum("tn,tnp->tp", C[:, 0], S) + 0.5 * xs[:, 0])
    # norms: unit root mean square, zero mean
    z = P.layer_norm(rng.standard_normal((3, 50)) + 4, np.ones(50), 0.0)
    assert np.allclose(z.mean(1), 0) and np.allclose((z * z).mean(1), 1)
    assert np.allclose((P.rms_norm(rng.standard_normal((3, 50)), np.ones(50), 0.0) ** 2).mean(1), 1)
    assert np.allclose(P.softplus(np.array([-800.0, 0.0, 800.0])), [0, np.log(2), 800])


def test_checkpoint_writer_round_trip(tmp_path):
    t = Y.random_tensors(CFG, 2)
    Y.write_checkpoint(tmp_path, CFG, t)
    raw = (tmp_path / "model.safetensors").read_bytes()
    n = struct.unpack("<Q", raw[:8])[0]
    head = json.loads(raw[8:8 + n])
    assert list(head) == list(Y.tensor_shapes(CFG)) == list(t)
    for k, h in head.items():
        lo, hi = h["data_offsets"]
        assert np.array_equal(Y.from_bf16(np.frombuffer(raw[8 + n + lo:8 + n + hi], np.uint16)).reshape(h["shape"]), t[k]), k
