"""Plain, slow numpy statements of the layer mechanisms that safetensors models are built from (the Dibosun design):
one function per mechanism, over whole sequences, in the precision of the arrays handed in. They share nothing with
the product path; the tests compare the engine with them."""

from __future__ import annotations

import numpy as np


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0) + np.log1p(np.exp(-np.abs(z)))


def relu_squared_ff(h, up, down):
    u = np.maximum(h @ up.T, 0)
    return (u * u) @ down.T


def latent_of(h, w, eps):
    """The cached latent of every token: [T, kv_rank]."""
    return rms_norm(h @ w["dkv"].T, w["dkv.norm"], eps)


def window_mask(n, size):
    """visible[i, j]: token i sees token j, itself and the size - 1 before it (size 0: everything before it)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i - j < size) if size else True)


def softmax_rows(s, visible):
    s = np.where(visible, s, -np.inf)
    p = np.exp(s - s.max(-1, keepdims=True))
    return p / p.sum(-1, keepdims=True)


def latent_attention(h, c, w, m, eps):
    """h: the mixer's input, c: the latents it attends to, m: its configuration."""
    T, H = h.shape[0], m["heads"]
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, m["dim"])
    k = (c @ w["uk"].T).reshape(T, H, m["dim"])
    v = (c @ w["uv"].T).reshape(T, H, m["vdim"])
    gate = sigmoid(h @ w["g"].T)
    visible = window_mask(T, (m.get("mask") or {}).get("size", 0))
    out = np.empty((T, H, m["vdim"]), h.dtype)
    for a in range(H):
        out[:, a] = softmax_rows(q[:, a] @ k[:, a].T * h.dtype.type(m["scale"]), visible) @ v[:, a] * gate[:, a:a + 1]
    return out.reshape(T, -1) @ w["o"].T


def causal_conv(x, taps, bias):
    """Per channel, the last column of taps at the current token, zeros before the start."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1]), x.dtype), x])
    return sum(padded[i:i + x.shape[0]] * taps[:, i] for i in range(n)) + bias


def ssd_scan(x, B, C, dt, A_log, D):
    """x [T, heads, P], B and C [T, groups, N], dt [T, heads] (after softplus) -> y [T, heads, P]."""
    T, H, P = x.shape
    per = H // B.shape[1]
    S = np.zeros((H, B.shape[2], P), x.dtype)
    y = np.empty_like(x)
    for t in range(T):
        Bh, Ch = np.repeat(B[t], per, 0), np.repeat(C[t], per, 0)
        S = np.exp(-np.exp(A_log) * dt[t])[:, None, None] * S + (dt[t][:, None] * Bh)[:, :, None] * x[t][:, None, :]
        y[t] = np.einsum("hnp,hn->hp", S, Ch) + D[:, None] * x[t]
    return y


def mamba2(h, w, m, eps):
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = np.split(h @ w["in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    y = ssd_scan(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    y = (y.reshape(T, inner) * silu(z)).reshape(T, m["norm_groups"], -1)
    y = rms_norm(y, w["norm"].reshape(m["norm_groups"], -1), eps).reshape(T, inner)
    return y @ w["o"].T


def layer_order(cfg):
    """(layer, whether the embedding output is added before it) of every layer run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    lo, hi = loop["start"], loop["stop"]
    order = [(i, False) for i in range(lo)]
    for turn in range(loop["times"]):
        order += [(i, turn > 0 and i == lo) for i in range(lo, hi)]
    return order + [(i, False) for i in range(hi, n)]


def run_stack(cfg, tensors, tokens, dtype=np.float64, keep=None):
    """Logits [T, vocab] of one sequence; keep: a list that receives the residual stream after every layer run."""
    W = {k: np.asarray(v, dtype) for k, v in tensors.items()}
    eps = dtype(cfg["norm"]["eps"])
    first = x = W["embed"][np.asarray(tokens)]
    latents = {}                                 # of a layer's latest pass
    for i, add_first in layer_order(cfg):
        p, layer = "l%d." % i, cfg["layers"][i]
        if add_first:
            x = x + first
        w = {k[len(p) + 4:]: v for k, v in W.items() if k.startswith(p + "mix.")}
        h = layer_norm(x, W[p + "norm1"], eps)
        m = layer["mixer"]
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                latents[i] = latent_of(h, w, eps)
            mix = latent_attention(h, latents[i if m.get("kv_from") is None else m["kv_from"]], w, m, eps)
        else:
            mix = mamba2(h, w, m, eps)
        add = mix * W[p + "ls1"]
        if layer.get("mlp"):
            add = add + relu_squared_ff(h, W[p + "mlp.up"], W[p + "mlp.down"]) * W[p + "ls2"]
        x = x + add
        if keep is not None:
            keep.append(x)
    return layer_norm(x, W["final.norm"], eps) @ W["embed"].T
