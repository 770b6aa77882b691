"""Plain, slow numpy statements of the mechanisms of the Vifanex design, one function each, over whole sequences, in the
precision of the arrays handed in. They share nothing with the product path; the tests compare the engine with them."""

from __future__ import annotations

import math

import numpy as np

from plain_layers import causal_conv, rms_norm, sigmoid, silu, softmax_rows, softplus, window_mask


def banded_frequencies(rot):
    """Radians per position of every rotated pair. Stretched rotation tells pairs apart by their wavelength: those that turn
    at least `high` times within the original length stay, those that turn at most `low` times slow down by the factor."""
    n = rot["dims"]
    out = []
    for i in range(n // 2):
        f = rot["base"] ** (-2.0 * i / n)
        s = rot.get("scaling")
        if s:
            turns = s["original"] * f / (2.0 * math.pi)
            share = min(max((turns - s["low"]) / (s["high"] - s["low"]), 0.0), 1.0)
            f = share * f + (1.0 - share) * f / s["factor"]
        out.append(f)
    return np.array(out)


def rotate_neighbours(x, positions, rot):
    """x [T, heads, dim]: the first rot.dims columns turned, pair i being columns 2 i and 2 i + 1."""
    n = rot["dims"]
    a = np.asarray(positions, np.float64)[:, None] * banded_frequencies(rot)[None, :]
    c, s = np.cos(a).astype(x.dtype)[:, None], np.sin(a).astype(x.dtype)[:, None]
    out = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def mixed_values(v, first, share):
    """Values of a layer beside those of the first layer that mixes."""
    return v + share * (first - v)


def windowed_attention(h, w, m, eps, first_values):
    """h [T, width] -> [T, width]. first_values: a list that the first mixing layer leaves its values in."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w["q"].T + w["q.b"], w["q.norm"], eps).reshape(T, H, D)
    k = rms_norm(h @ w["k"].T + w["k.b"], w["k.norm"], eps).reshape(T, G, D)
    v = h @ w["v"].T + w["v.b"]
    if m.get("v_mix"):
        if first_values:
            v = mixed_values(v, first_values[0], w["vmix"])
        else:
            first_values.append(v)
    v = v.reshape(T, G, V)
    if m.get("rot"):
        q, k = rotate_neighbours(q, range(T), m["rot"]), rotate_neighbours(k, range(T), m["rot"])
    visible = window_mask(T, (m.get("mask") or {}).get("size", 0))
    out = np.empty((T, H, V), h.dtype)
    for a in range(H):
        g = a // (H // G)
        out[:, a] = softmax_rows(q[:, a] @ k[:, g].T * h.dtype.type(m["scale"]), visible) @ v[:, g]
    return out.reshape(T, H * V) @ w["o"].T


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def channel_delta_scan(q, k, v, beta, g):
    """q, k, g [T, heads, D], v [T, heads, V], beta [T, heads] -> the read-outs [T, heads, V]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]), v.dtype)
    out = np.empty_like(v)
    for t in range(T):
        S = S * g[t][:, :, None]
        held = np.einsum("hdv,hd->hv", S, k[t])
        S = S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - held))[:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def channel_decay(a, A_log, dt_bias, heads):
    """a [T, heads * D] -> the factor per token, head and key channel."""
    rate = np.exp(A_log)[None, :, None]
    return np.exp(-rate * softplus(a + dt_bias).reshape(len(a), heads, -1))


def channel_delta(h, w, m, eps):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"], 0)) for n in ("q", "k", "v"))
    per = H // G
    q = np.repeat(unit(q.reshape(T, G, D)) * h.dtype.type(D) ** -0.5, per, axis=1)
    k = np.repeat(unit(k.reshape(T, G, D)), per, axis=1)
    g = channel_decay(h @ w["a1"].T @ w["a2"].T, w["A_log"], w["dt_bias"], H)
    o = channel_delta_scan(q, k, v.reshape(T, H, V), sigmoid(h @ w["b"].T), g)
    o = rms_norm(o, w["norm"], eps) * sigmoid(h @ w["g1"].T @ w["g2"].T).reshape(T, H, V)
    return o.reshape(T, H * V) @ w["o"].T


def clamped_ff(h, gate, up, down, limit, gate_b=0.0, up_b=0.0, down_b=0.0):
    z = np.minimum(h @ gate.T + gate_b, limit)
    u = np.clip(h @ up.T + up_b, -limit, limit)
    return (z * sigmoid(1.702 * z) * (u + 1.0)) @ down.T + down_b


def allowed_experts(s, groups):
    """Scores [T, experts] -> which experts belong to a kept group (groups of neighbours, ranked by their largest score)."""
    if not groups:
        return np.ones(s.shape, bool)
    T, n = s.shape
    best = s.reshape(T, groups["count"], -1).max(-1)
    kept = np.zeros(best.shape, bool)
    np.put_along_axis(kept, np.argsort(-best, axis=1, kind="stable")[:, :groups["keep"]], True, 1)
    return np.repeat(kept, n // groups["count"], axis=1)


def choose_experts(z, router):
    """Logits [T, experts] -> chosen experts [T, top] and their weights: softmax over all experts, not renormalized."""
    e = np.exp(z - z.max(1, keepdims=True))
    s = e / e.sum(1, keepdims=True)
    ranked = np.where(allowed_experts(s, router.get("groups")), s, -1.0)
    sel = np.argsort(-ranked, axis=1, kind="stable")[:, :router["top"]]
    return sel, np.take_along_axis(s, sel, 1) * router.get("scale", 1.0)


def routing_lead(z, router):
    """By how much every token's choice is decided, in logits: of groups, and of experts within the kept ones."""
    T, n = z.shape
    lead = np.full(T, np.inf)
    groups = router.get("groups")
    if groups and groups["keep"] < groups["count"]:
        best = np.sort(z.reshape(T, groups["count"], -1).max(-1), axis=1)[:, ::-1]
        lead = best[:, groups["keep"] - 1] - best[:, groups["keep"]]
    s = np.sort(np.where(allowed_experts(z, groups), z, -np.inf), axis=1)[:, ::-1]
    top = router["top"]
    return np.minimum(lead, s[:, top - 1] - s[:, top]) if top < n else lead


def expert_ff(h, w, mlp):
    sel, weight = choose_experts(h @ w["router"].T, mlp["router"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(sel[t], weight[t]):
            n = "e%d." % e
            out[t] += p * clamped_ff(h[t:t + 1], w[n + "gate"], w[n + "up"], w[n + "down"], mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out = out + clamped_ff(h, w["shared.gate"], w["shared.up"], w["shared.down"], mlp["shared"]["limit"])
    return out


def streams_in(xs, w):
    """What a sublayer reads of the streams [s, T, width]."""
    return np.einsum("s,ste->te", w["in"], xs)


def streams_out(xs, y, w):
    """The streams after a sublayer's output y; w.mix is [from, to]."""
    return np.einsum("st,sne->tne", w["mix"], xs) + w["out"][:, None, None] * y[None]


def run_stack(cfg, tensors, tokens, dtype=np.float64, keep=None, leads=None):
    """Logits [T, vocab] of one sequence; keep: a list that receives the sum of the streams after every layer, leads one
    that receives the routing's leads of every layer with experts."""
    W = {k: np.asarray(v, dtype) for k, v in tensors.items()}
    eps = dtype(cfg["norm"]["eps"])
    xs = np.repeat((W["embed"][np.asarray(tokens)] * dtype(cfg["embedding"]["scale"]))[None], cfg["streams"], axis=0)
    first_values = []
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % i
        part = lambda name: {k[len(p + name):]: v for k, v in W.items() if k.startswith(p + name)}
        hc = part("hc1.")
        h = rms_norm(streams_in(xs, hc), W[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = windowed_attention(h, part("mix."), layer["mixer"], eps, first_values)
        else:
            y = channel_delta(h, part("mix."), layer["mixer"], eps)
        xs = streams_out(xs, y, hc)
        mlp = layer.get("mlp")
        if mlp:
            hc = part("hc2.")
            h, w = rms_norm(streams_in(xs, hc), W[p + "norm2"], eps), part("mlp.")
            if mlp["kind"] == "dense":
                y = clamped_ff(h, w["gate"], w["up"], w["down"], mlp["limit"], w["gate.b"], w["up.b"], w["down.b"])
            else:
                if leads is not None:
                    leads.append(routing_lead(h @ w["router"].T, mlp["router"]))
                y = expert_ff(h, w, mlp)
            xs = streams_out(xs, y, hc)
        if keep is not None:
            keep.append(xs.sum(0))
    z = rms_norm(xs.sum(0), W["final.norm"], eps) @ W["head"].T
    cap = cfg.get("logit_softcap")
    return cap * np.tanh(z / cap) if cap else z
