"""Random-weight checkpoint folders (config.json + model.safetensors) of layer-stack models, for benchmarks and tests:
the tensors a configuration asks for, values that keep activations of order one, and the safetensors writer."""

from __future__ import annotations

import json
import struct
from pathlib import Path

import numpy as np


def latent_layer(heads, dim, vdim, q_rank, kv_rank, window, ff, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": window}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mamba2_layer(heads, vdim, state, groups, conv, norm_groups, ff):
    m = {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}
    return {"type": "mamba2", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def dibosun(width, vocab, layers, eps=1e-5):
    return {"architecture": "Dibosun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


def rotary(dims, base=10000.0, factor=None, original=64, fast=32.0, slow=1.0):
    r = {"dims": dims, "base": base}
    if factor is not None:
        r["scaling"] = {"factor": factor, "original": original, "fast": fast, "slow": slow}
    return r


def dense_mlp(ff):
    return {"kind": "dense", "ff": ff}


def moe_mlp(experts, top, ff, shared_ff=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared_ff is not None:
        out["shared"] = {"ff": shared_ff}
    return out


def attention_layer(heads, kv_heads, dim, mask, rot, mlp, scale=None, softcap=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": mask}, "rot": rot,
         "scale": dim ** -0.5 if scale is None else scale}
    if softcap is not None:
        m["softcap"] = softcap
    return {"type": "attention", "mixer": m, "mlp": mlp}


def pomisun(width, vocab, layers, eps=1e-5, loop=None):
    """loop: (start, stop, times) of the layers that run several times, or none."""
    out = {"architecture": "Pomisun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def banded_rotary(dims, base=10000.0, factor=None, original=64, high=4.0, low=1.0):
    r = {"dims": dims, "base": base}
    if factor is not None:
        r["scaling"] = {"factor": factor, "original": original, "high": high, "low": low}
    return r


def clamped_mlp(ff, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def clamped_moe(experts, top, ff, limit=1.5, shared=None, groups=None, scale=1.0):
    """shared: (width, limit) of the shared expert; groups: (count, kept)."""
    router = {"experts": experts, "top": top, "scale": scale}
    if groups:
        router["groups"] = dict(zip(("count", "keep"), groups))
    out = {"kind": "moe", "router": router, "expert": {"ff": ff, "limit": limit}}
    if shared:
        out["shared"] = dict(zip(("ff", "limit"), shared))
    return out


def normed_attention_layer(heads, kv_heads, dim, vdim, window, rot, mlp, scale=None, v_mix=False):
    """Grouped attention with values of its own, biases, and queries and keys normed over all their heads."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window} if window else None, "rot": rot,
         "scale": dim ** -0.5 if scale is None else scale, "v_mix": v_mix}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def channel_delta_layer(heads, kv_heads, dim, vdim, conv, mlp, decay_rank, gate_rank):
    """The two inner widths are what the tensors get; the engine takes them from there."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "decay_rank": decay_rank, "gate_rank": gate_rank}
    return {"type": "channel_delta", "mixer": m, "mlp": mlp}


def vifanex(width, vocab, layers, streams=2, eps=1e-5, softcap=20.0, embedding_scale=1.0):
    return {"architecture": "Vifanex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "streams": streams, "layers": layers,
            "logit_softcap": softcap, "embedding": {"scale": embedding_scale}}


def parallel_mixer_layer(attention, mamba2, scales, rot, mlp, scale=None):
    """Attention (heads, kv_heads, dim, vdim) and Mamba-2 (heads, vdim, state, groups, conv, norm_groups) over one input."""
    left = dict(zip(("heads", "kv_heads", "dim", "vdim"), attention), rot=rot, scale=attention[2] ** -0.5 if scale is None else scale)
    right = dict(zip(("heads", "vdim", "state", "groups", "conv", "norm_groups"), mamba2))
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]}, "mlp": mlp}


def hgrn2_layer(heads, dim, vdim, mlp):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": mlp}


def delta_layer(heads, kv_heads, dim, vdim, conv, mlp):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def kilurax(width, vocab, layers, groups=2, taps=3, residual=0.7, eps=1e-5, embedding_scale=2.0, pairs=(97, 31, 5)):
    """pairs: buckets and the two factors of the embedding of neighbouring tokens."""
    return {"architecture": "Kilurax", "width": width, "vocab": vocab, "norm": {"eps": eps, "groups": groups}, "canon": {"taps": taps},
            "residual_mult": residual, "embedding": {"scale": embedding_scale, "bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), pairs))}, "layers": layers}


def _kilurax_shapes(cfg) -> dict:
    E = cfg["width"]
    out = {"embed": (cfg["vocab"], E), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, E), "embed.norm": (E,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = "l%d." % i, layer["mixer"], layer.get("mlp")
        x = p + "mix."
        for q in ("1", "2") if mlp else ("1",):
            out.update({p + "norm" + q: (E,), p + "norm" + q + "b": (E,), p + "canon" + q: (E, cfg["canon"]["taps"])})
        if layer["type"] == "parallel":
            a, s = m["left"], m["right"]
            for name, n in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                out.update({x + "left." + name: (n, E), x + "left." + name + ".b": (n,)})
            out.update({x + "left.o": (E, a["heads"] * a["vdim"]), x + "left.o.b": (E,)})
            out.update(_mamba2_shapes(x + "right.", s, E))
        elif layer["type"] == "hgrn2":
            H, D, V = m["heads"], m["dim"], m["vdim"]
            out.update({x + "q": (H * D, E), x + "f": (H * D, E), x + "f.b": (H * D,), x + "lower": (H * D,), x + "v": (H * V, E), x + "norm": (V,), x + "o": (E, H * V)})
        else:
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for name, n in (("q", G * D), ("k", G * D), ("v", H * V)):
                out.update({x + name: (n, E), x + name + ".conv": (n, m["conv"])})
            out.update({x + "b": (H, E), x + "A_log": (H,), x + "norm": (V,), x + "a": (H, E), x + "dt_bias": (H,), x + "g": (H * V, E), x + "o": (E, H * V)})
        if not mlp:
            continue
        out[p + "mlp.router"] = (mlp["router"]["experts"], E)
        for e in range(mlp["router"]["experts"]):
            out.update(_gated_shapes(p + "mlp.e%d." % e, mlp["expert"]["ff"], E))
        if mlp.get("shared"):
            out.update(_gated_shapes(p + "mlp.shared.", mlp["shared"]["ff"], E))
    out["final.norm"] = (E,)
    out["head"] = (cfg["vocab"], E)
    return out


def _mamba2_shapes(p, m, E):
    inner, bc = m["heads"] * m["vdim"], 2 * m["groups"] * m["state"]
    out = {p + "in": (2 * inner + bc + m["heads"], E), p + "conv": (inner + bc, m["conv"]), p + "conv.b": (inner + bc,)}
    out.update({p + name: (m["heads"],) for name in ("dt_bias", "A_log", "D")})
    out.update({p + "norm": (inner,), p + "o": (E, inner)})
    return out


def _vifanex_shapes(cfg) -> dict:
    E, s = cfg["width"], cfg["streams"]
    out = {"embed": (cfg["vocab"], E)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = "l%d." % i, layer["mixer"], layer.get("mlp")
        x, H, G, D, V = p + "mix.", m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for q in (1, 2) if mlp else (1,):
            out[p + "norm%d" % q] = (E,)
            out.update({p + "hc%d.in" % q: (s,), p + "hc%d.out" % q: (s,), p + "hc%d.mix" % q: (s, s)})
        if layer["type"] == "attention":
            for name, n in (("q", H * D), ("k", G * D), ("v", G * V)):
                out[x + name] = (n, E)
                out[x + name + ".b"] = (n,)
            out[x + "q.norm"], out[x + "k.norm"] = (H * D,), (G * D,)
            if m["v_mix"]:
                out[x + "vmix"] = ()
        else:
            for name, n in (("q", G * D), ("k", G * D), ("v", H * V)):
                out[x + name] = (n, E)
                out[x + name + ".conv"] = (n, m["conv"])
            out.update({x + "b": (H, E), x + "A_log": (H,), x + "norm": (V,), x + "a1": (m["decay_rank"], E), x + "a2": (H * D, m["decay_rank"]),
                        x + "dt_bias": (H * D,), x + "g1": (m["gate_rank"], E), x + "g2": (H * V, m["gate_rank"])})
        out[x + "o"] = (E, H * V)
        if not mlp:
            continue
        if mlp["kind"] == "dense":
            out.update(_gated_shapes(p + "mlp.", mlp["ff"], E))
            out.update({p + "mlp.gate.b": (mlp["ff"],), p + "mlp.up.b": (mlp["ff"],), p + "mlp.down.b": (E,)})
            continue
        out[p + "mlp.router"] = (mlp["router"]["experts"], E)
        for e in range(mlp["router"]["experts"]):
            out.update(_gated_shapes(p + "mlp.e%d." % e, mlp["expert"]["ff"], E))
        if mlp.get("shared"):
            out.update(_gated_shapes(p + "mlp.shared.", mlp["shared"]["ff"], E))
    out["final.norm"] = (E,)
    out["head"] = (cfg["vocab"], E)
    return out


def _gated_shapes(p, ff, E):
    return {p + "gate": (ff, E), p + "up": (ff, E), p + "down": (E, ff)}


def tensor_shapes(cfg) -> dict:
    E = cfg["width"]
    out = {"embed": (cfg["vocab"], E)}
    if cfg["architecture"] == "Vifanex":
        return _vifanex_shapes(cfg)
    if cfg["architecture"] == "Kilurax":
        return _kilurax_shapes(cfg)
    if cfg["architecture"] == "Pomisun":
        for i, layer in enumerate(cfg["layers"]):
            p, m, mlp = "l%d." % i, layer["mixer"], layer.get("mlp")
            out[p + "norm1"] = (E,)
            out[p + "mix.q"] = (m["heads"] * m["dim"], E)
            out[p + "mix.k"] = (m["kv_heads"] * m["dim"], E)
            out[p + "mix.o"] = (E, m["heads"] * m["dim"])
            if not mlp:
                continue
            out[p + "norm2"] = (E,)
            if mlp["kind"] == "dense":
                out.update(_gated_shapes(p + "mlp.", mlp["ff"], E))
                continue
            out[p + "mlp.router"] = (mlp["router"]["experts"], E)
            for e in range(mlp["router"]["experts"]):
                out.update(_gated_shapes(p + "mlp.e%d." % e, mlp["expert"]["ff"], E))
            if mlp.get("shared"):
                out.update(_gated_shapes(p + "mlp.shared.", mlp["shared"]["ff"], E))
                out[p + "mlp.shared.sg"] = (1, E)
        out["final.norm"] = (E,)
        return out
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        out[p + "norm1"] = (E,)
        if layer["type"] == "latent_attention":
            H = m["heads"]
            out[p + "mix.dq"] = (m["q_rank"], E)
            out[p + "mix.dq.norm"] = (m["q_rank"],)
            out[p + "mix.uq"] = (H * m["dim"], m["q_rank"])
            if m.get("kv_from") is None:
                out[p + "mix.dkv"] = (m["kv_rank"], E)
                out[p + "mix.dkv.norm"] = (m["kv_rank"],)
            out[p + "mix.uk"] = (H * m["dim"], m["kv_rank"])
            out[p + "mix.uv"] = (H * m["vdim"], m["kv_rank"])
            out[p + "mix.g"] = (H, E)
            out[p + "mix.o"] = (E, H * m["vdim"])
        else:
            out.update(_mamba2_shapes(p + "mix.", m, E))
        out[p + "ls1"] = (E,)
        if layer.get("mlp"):
            out[p + "mlp.up"] = (layer["mlp"]["ff"], E)
            out[p + "mlp.down"] = (E, layer["mlp"]["ff"])
            out[p + "ls2"] = (E,)
    out["final.norm"] = (E,)
    return out


def mean_and_std(name, shape, architecture="Dibosun"):
    """Of a tensor's normal distribution."""
    leaf = name.rsplit(".", 1)[-1]
    if architecture == "Pomisun" and leaf.startswith("norm"):
        return -0.1, 0.2                     # stored as the difference from one
    if architecture == "Vifanex":
        if ".hc" in name:
            return (0.8, 0.3) if leaf == "out" else (1.0 / shape[0], 0.3)
        if leaf == "vmix":
            return 0.5, 0.3
        if len(shape) == 2 and leaf == "b":
            return 0.0, shape[-1] ** -0.5
        if leaf == "b":
            return 0.0, 0.3
    if architecture == "Kilurax":
        if leaf == "lower":
            return 0.4, 0.3                  # clipped to what a lower bound may be
        if name.endswith(".f.b"):
            return 2.0, 1.5
        if leaf.startswith("canon"):
            return 0.0, 0.3
        if leaf == "b" and len(shape) == 2:
            return 0.0, shape[-1] ** -0.5
        if name == "bigram":
            return 0.0, 1.0
        if leaf == "b" and ".left." in name:
            return 0.0, 0.3
    if leaf == "router":
        return 0.0, 2.0 * shape[-1] ** -0.5
    if leaf == "dt_bias":
        return -2.0, 0.7
    if leaf == "A_log":
        return -0.5, 1.0
    if leaf == "D" or leaf == "norm" or leaf.startswith("norm") or leaf.startswith("ls"):
        return 0.9, 0.2
    if leaf == "b":
        return 0.0, 0.1
    if leaf == "conv":
        return 0.0, 0.5
    if name == "embed":
        return 0.0, 1.0
    return 0.0, shape[-1] ** -0.5


def _header(items):
    head, at = {}, 0
    for name, shape in items.items():
        n = 2 * int(np.prod(shape))
        head[name] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [at, at + n]}
        at += n
    raw = json.dumps(head).encode()
    raw += b" " * (-len(raw) % 8)
    return struct.pack("<Q", len(raw)) + raw


def to_bf16(x) -> np.ndarray:
    """f32 -> bf16 bits, to nearest even."""
    b = np.ascontiguousarray(x, np.float32).view(np.uint32).astype(np.uint64)
    return ((b + 0x7FFF + ((b >> 16) & 1)) >> 16).astype(np.uint16).reshape(np.shape(x))


def from_bf16(b) -> np.ndarray:
    return (np.atleast_1d(np.asarray(b, np.uint32)) << 16).view(np.float32).reshape(np.shape(b))


def random_tensors(cfg, seed) -> dict:
    """name -> f32 array whose values are exact in bf16."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        mean, std = mean_and_std(name, shape, cfg["architecture"])
        v = mean + std * rng.standard_normal(shape)
        out[name] = from_bf16(to_bf16(np.clip(v, 0.0, 1.0) if name.endswith(".lower") else v))
    return out


def write_checkpoint(folder, cfg, tensors) -> Path:
    """The folder with the given tensors (values exact in bf16)."""
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    with open(folder / "model.safetensors", "wb") as f:
        f.write(_header({k: v.shape for k, v in tensors.items()}))
        for v in tensors.values():
            f.write(to_bf16(v).tobytes())
    return folder


def write_random_checkpoint(folder, cfg, seed, device="cuda") -> Path:
    """A large random checkpoint, generated tensor by tensor with torch."""
    import torch

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    gen = torch.Generator(device=device).manual_seed(seed)
    shapes = tensor_shapes(cfg)
    with open(folder / "model.safetensors", "wb") as f:
        f.write(_header(shapes))
        for name, shape in shapes.items():
            mean, std = mean_and_std(name, shape, cfg["architecture"])
            t = torch.empty(shape, device=device, dtype=torch.float32).normal_(mean, std, generator=gen)
            t = (t.clamp_(0.0, 1.0) if name.endswith(".lower") else t).to(torch.bfloat16)
            f.write(t.view(torch.int16).cpu().numpy().tobytes())
    return folder


def matrix_bytes(cfg) -> int:
    """Bytes of the matrices one step streams (the embedding counted once, as the output head)."""
    return sum(2 * int(np.prod(s)) for n, s in tensor_shapes(cfg).items() if len(s) == 2 and not n.endswith(".conv") and ".canon" not in n and n != "bigram")
