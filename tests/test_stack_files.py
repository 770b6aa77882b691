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


@pytest.mark.parametrize("edit, message", [
    (lambda c: c.update(architecture="Other"), "unsupported model architecture: Other"),
    (lambda c: c.pop("width"), "lacks 'width'"),
    (lambda c: c.update(vocab=3.5), "'vocab' is no size"),
    (lambda c: c.update(layers=[]), "1 to 4096 layers"),
    (lambda c: c["layers"][0].update(type="attention"), "unknown layer type 'attention'"),
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
