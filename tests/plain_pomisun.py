"""Plain, slow numpy statements of the mechanisms of the Pomisun design, one function each, over whole sequences, in the
precision of the arrays handed in. They share nothing with the product path; the tests compare the engine with them."""

from __future__ import annotations

import math

import numpy as np

from plain_layers import layer_order, sigmoid, silu, softmax_rows


def gelu_tanh(z):
    return z * 0.5 * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms_norm_around_one(x, w, eps):
    """Root-mean-square norm whose weight is stored as its difference from one."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * (1.0 + w)


def yarn_frequencies(rot):
    """Radians per position of every rotated pair, and the factor on cosines and sines."""
    n, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if not s:
        return np.array(plain), 1.0

    def place(turns):      # the (fractional) pair that turns this often within the original length
        return n * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(place(s["fast"])), 0), min(math.ceil(place(s["slow"])), n - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1.0 - ramp))
    return np.array(out), 0.1 * math.log(s["factor"]) + 1.0


def rotate_half(x, positions, rot):
    """x [T, heads, dim]: the first rot.dims columns turned, pair i being columns i and i + dims / 2."""
    freq, magnitude = yarn_frequencies(rot)
    half = rot["dims"] // 2
    a = np.asarray(positions, np.float64)[:, None] * freq[None, :]
    c, s = (np.cos(a) * magnitude).astype(x.dtype)[:, None], (np.sin(a) * magnitude).astype(x.dtype)[:, None]
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * half:]], axis=-1)


def chunk_mask(n, size):
    """visible[i, j]: token i sees the tokens of its own chunk up to itself (size 0: everything before it)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i // size == j // size) if size else True)


def soft_capped(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def attention_scores(q, k, scale, cap):
    return soft_capped(q @ k.T * scale, cap)


def grouped_attention(h, w, m):
    """h [T, width] -> [T, width]; the values are the keys before their rotation."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w["q"].T).reshape(T, H, D)
    v = (h @ w["k"].T).reshape(T, G, D)
    q, k = rotate_half(q, range(T), m["rot"]), rotate_half(v, range(T), m["rot"])
    visible = chunk_mask(T, (m.get("mask") or {}).get("size", 0))
    out = np.empty((T, H, D), h.dtype)
    for a in range(H):
        g = a // (H // G)
        s = attention_scores(q[:, a], k[:, g], h.dtype.type(m["scale"]), m.get("softcap"))
        out[:, a] = softmax_rows(s, visible) @ v[:, g]
    return out.reshape(T, H * D) @ w["o"].T


def gated_ff(h, gate, up, down, act):
    return (act(h @ gate.T) * (h @ up.T)) @ down.T


def choose_experts(z, top):
    """Logits [T, experts] -> chosen experts [T, top] and their weights, the softmax over the chosen logits."""
    sel = np.argsort(-z, axis=1, kind="stable")[:, :top]
    e = np.take_along_axis(z, sel, 1)
    e = np.exp(e - e.max(1, keepdims=True))
    return sel, e / e.sum(1, keepdims=True)


def expert_ff(h, w, mlp):
    sel, weight = choose_experts(h @ w["router"].T, mlp["router"]["top"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(sel[t], weight[t]):
            n = "e%d." % e
            out[t] += p * gated_ff(h[t:t + 1], w[n + "gate"], w[n + "up"], w[n + "down"], silu)[0]
    if mlp.get("shared"):
        s = gated_ff(h, w["shared.gate"], w["shared.up"], w["shared.down"], silu)
        out = out + s * sigmoid(h @ w["shared.sg"].T)
    return out


def routing_lead(z, top):
    """By how much the last chosen logit of every token exceeds the next."""
    s = np.sort(z, axis=1)[:, ::-1]
    return s[:, top - 1] - s[:, top] if top < z.shape[1] else np.full(len(z), np.inf)


def run_stack(cfg, tensors, tokens, dtype=np.float64, keep=None, leads=None):
    """Logits [T, vocab] of one sequence; keep: a list that receives the residual stream after every layer run, leads one
    that receives the routing's leads of every layer with experts."""
    W = {k: np.asarray(v, dtype) for k, v in tensors.items()}
    eps = dtype(cfg["norm"]["eps"])
    first = x = W["embed"][np.asarray(tokens)]
    for i, add_first in layer_order(cfg):
        p, layer = "l%d." % i, cfg["layers"][i]
        part = lambda name: {k[len(p + name):]: v for k, v in W.items() if k.startswith(p + name)}
        if add_first:
            x = x + first
        x = x + grouped_attention(rms_norm_around_one(x, W[p + "norm1"], eps), part("mix."), layer["mixer"])
        if layer.get("mlp"):
            h, w = rms_norm_around_one(x, W[p + "norm2"], eps), part("mlp.")
            if leads is not None and layer["mlp"]["kind"] == "moe":
                leads.append(routing_lead(h @ w["router"].T, layer["mlp"]["router"]["top"]))
            x = x + (gated_ff(h, w["gate"], w["up"], w["down"], gelu_tanh) if layer["mlp"]["kind"] == "dense" else expert_ff(h, w, layer["mlp"]))
        if keep is not None:
            keep.append(x)
    return rms_norm_around_one(x, W["final.norm"], eps) @ W["embed"].T
