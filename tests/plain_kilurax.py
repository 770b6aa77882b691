"""Plain, slow numpy statements of the mechanisms of the Kilurax design, one function each, over whole sequences, in the
precision of the arrays handed in. They share nothing with the product path; the tests compare the engine with them."""

from __future__ import annotations

import numpy as np

from plain_layers import causal_conv, sigmoid, silu, softmax_rows, softplus, ssd_scan, window_mask


def grouped_norm(x, w, eps, groups):
    """Each of the equal consecutive parts of the last axis by its own root mean square, then the weight."""
    parts = x.reshape(*x.shape[:-1], groups, -1)
    parts = parts / np.sqrt((parts * parts).mean(-1, keepdims=True) + eps)
    return parts.reshape(x.shape) * w


def bigram_rows(tokens, b):
    """Row of the pair table for every token; a sequence's first token has the row behind the hashed ones."""
    tokens = [int(t) for t in tokens]
    return [b["buckets"]] + [(p * b["mul_prev"] + t * b["mul_cur"]) % b["buckets"] for p, t in zip(tokens, tokens[1:])]


def embed(tokens, W, cfg, eps):
    e = cfg["embedding"]
    x = W["embed"][np.asarray(tokens)] * W["embed"].dtype.type(e["scale"])
    x = x + W["bigram"][bigram_rows(tokens, e["bigram"])]
    return grouped_norm(x, W["embed.norm"], eps, cfg["norm"]["groups"])


def with_neighbours(h, taps):
    """What a sublayer reads: h and a convolution of it over the tokens up to its own."""
    return h + causal_conv(h, taps, 0)


def rotate_halves(x, rot):
    """x [T, heads, dim] at positions 0 ..: column i turns with column i + dims / 2."""
    n = rot["dims"]
    half = n // 2
    f = np.array([float(rot["base"]) ** (-2.0 * i / n) for i in range(half)])
    a = np.arange(len(x), dtype=np.float64)[:, None] * f
    c, s = np.cos(a).astype(x.dtype)[:, None], np.sin(a).astype(x.dtype)[:, None]
    u, v = x[..., :half], x[..., half:n]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., n:]], axis=-1)


def biased_attention(h, w, m):
    """Causal grouped attention with values of their own and biases on all four projections."""
    T, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = ((h @ w[n].T + w[n + ".b"]).reshape(T, heads, -1) for n, heads in (("q", H), ("k", G), ("v", G)))
    if m.get("rot"):
        q, k = rotate_halves(q, m["rot"]), rotate_halves(k, m["rot"])
    visible = window_mask(T, 0)
    out = np.empty((T, H, V), h.dtype)
    for a in range(H):
        g = a // (H // G)
        out[:, a] = softmax_rows(q[:, a] @ k[:, g].T * h.dtype.type(m["scale"]), visible) @ v[:, g]
    return out.reshape(T, H * V) @ w["o"].T + w["o.b"]


def state_space(h, w, m, eps):
    T, H, P, N, G = len(h), m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    p = h @ w["in"].T
    z, xbc, dt = p[:, :inner], p[:, inner:2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = xbc[:, :inner], xbc[:, inner:inner + G * N], xbc[:, inner + G * N:]
    y = ssd_scan(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    return grouped_norm(y.reshape(T, inner) * silu(z), w["norm"], eps, m["norm_groups"]) @ w["o"].T


def side_by_side(h, w, m, eps):
    part = lambda p: {k[len(p):]: v for k, v in w.items() if k.startswith(p)}
    t = h.dtype.type
    return t(m["left_scale"]) * biased_attention(h, part("left."), m["left"]) + t(m["right_scale"]) * state_space(h, part("right."), m["right"], eps)


def forget_scan(q, f, v):
    """q, f [T, heads, D], v [T, heads, V]: what a channel forgets is what it writes."""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2]), v.dtype)
    out = np.empty_like(v)
    for t in range(len(q)):
        S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def head_norm(o, w, eps):
    return o / np.sqrt((o * o).mean(-1, keepdims=True) + eps) * w


def forget_gate(z, lower):
    return lower + (1 - lower) * sigmoid(z)


def hgrn2(h, w, m, eps):
    T, H = len(h), m["heads"]
    q = silu(h @ w["q"].T).reshape(T, H, -1)
    f = forget_gate(h @ w["f"].T + w["f.b"], w["lower"]).reshape(T, H, -1)
    o = head_norm(forget_scan(q, f, (h @ w["v"].T).reshape(T, H, -1)), w["norm"], eps)
    return o.reshape(T, -1) @ w["o"].T


def delta_scan(q, k, v, beta, g):
    """q, k [T, heads, D], v [T, heads, V], beta, g [T, heads] -> the read-outs."""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2]), v.dtype)
    out = np.empty_like(v)
    for t in range(len(q)):
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def head_decay(a, A_log, dt_bias):
    return np.exp(-np.exp(A_log) * softplus(a + dt_bias))


def delta(h, w, m, eps):
    T, H, G, D = len(h), m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"], 0)) for n in ("q", "k", "v"))
    q = np.repeat(unit(q.reshape(T, G, D)) * h.dtype.type(D) ** -0.5, H // G, axis=1)
    k = np.repeat(unit(k.reshape(T, G, D)), H // G, axis=1)
    o = delta_scan(q, k, v.reshape(T, H, -1), sigmoid(h @ w["b"].T), head_decay(h @ w["a"].T, w["A_log"], w["dt_bias"]))
    o = head_norm(o, w["norm"], eps) * silu(h @ w["g"].T).reshape(T, H, -1)
    return o.reshape(T, -1) @ w["o"].T


def gated_ff(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def choose_experts(z, top):
    """Logits [T, experts] -> the chosen experts and their scores."""
    sel = np.argsort(-z, axis=1, kind="stable")[:, :top]
    return sel, sigmoid(np.take_along_axis(z, sel, 1))


def routing_lead(z, top):
    s = np.sort(z, axis=1)[:, ::-1]
    return s[:, top - 1] - s[:, top] if top < z.shape[1] else np.full(len(z), np.inf)


def expert_ff(h, w, mlp):
    sel, score = choose_experts(h @ w["router"].T, mlp["router"]["top"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, s in zip(sel[t], score[t]):
            n = "e%d." % e
            out[t] += gated_ff(s * h[t:t + 1], w[n + "gate"], w[n + "up"], w[n + "down"])[0]
    if mlp.get("shared"):
        out = out + gated_ff(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


MIXERS = {"parallel": side_by_side, "hgrn2": hgrn2, "delta": delta}


def run_stack(cfg, tensors, tokens, dtype=np.float64, keep=None, leads=None):
    """Logits [T, vocab] of one sequence; keep: a list that receives the residual stream after every layer, leads one that
    receives the routing's leads of every layer with experts."""
    W = {k: np.asarray(v, dtype) for k, v in tensors.items()}
    eps, m, groups = dtype(cfg["norm"]["eps"]), dtype(cfg["residual_mult"]), cfg["norm"]["groups"]
    norm = lambda x, name: grouped_norm(x, W[name], eps, groups)
    x = embed(tokens, W, cfg, eps)
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % i
        part = lambda name: {k[len(p + name):]: v for k, v in W.items() if k.startswith(p + name)}
        h = with_neighbours(norm(x, p + "norm1"), W[p + "canon1"])
        x = x + m * norm(MIXERS[layer["type"]](h, part("mix."), layer["mixer"], eps), p + "norm1b")
        if layer.get("mlp"):
            h, w = with_neighbours(norm(x, p + "norm2"), W[p + "canon2"]), part("mlp.")
            if leads is not None:
                leads.append(routing_lead(h @ w["router"].T, layer["mlp"]["router"]["top"]))
            x = x + m * norm(expert_ff(h, w, layer["mlp"]), p + "norm2b")
        if keep is not None:
            keep.append(x)
    return norm(x, "final.norm") @ W["head"].T
