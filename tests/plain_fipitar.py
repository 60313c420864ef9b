"""A plain, slow implementation of the Fipitar design in float64 numpy, one function per mechanism.

Everything is written from the design's equations and shares no code with the package: whole
sequences at once, no cache, no batching.  ``forward`` takes a config.json dictionary and the
tensors by their file names.

Notation: ``x`` [T, W] the residual stream of one sequence, which the sublayers read as it is (``h``), ``eps`` the
norms' constant, ``t`` the tensors by file name, ``p`` the prefix of a mixer's or feed-forward's tensors, ``m`` the
mixer's (or feed-forward's) object of config.json.  Linear weights are ``[out, in]`` and applied as ``h @ W.T``.
"""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def layer_norm(x, w, b, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


# ---------------------------------------------------------------- positions
def frequencies(rot):
    """``(f, magnitude)``: the frequency of every rotated pair and the factor on all cosines and sines."""
    base, dims, s = float(rot["base"]), rot["dims"], rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not s:
        return f, 1.0
    index = lambda turns: dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(index(s["fast"])), 0), min(math.ceil(index(s["slow"])), dims - 1)
    out = []
    for i, v in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(v / s["factor"] * ramp + v * (1.0 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate(v, rot, interleaved):
    """The first rot.dims of the last axis of v [T, ..., D] turned by position (row number): pairs (2i, 2i + 1) or
    (i, i + dims / 2)."""
    f, magnitude = frequencies(rot)
    dims = rot["dims"]
    a = np.arange(v.shape[0], dtype=np.float64)[:, None] * np.array(f)
    a = a.reshape(v.shape[0], *([1] * (v.ndim - 2)), dims // 2)
    c, s = magnitude * np.cos(a), magnitude * np.sin(a)
    first, second = (np.arange(0, dims, 2), np.arange(1, dims, 2)) if interleaved else (np.arange(dims // 2), np.arange(dims // 2, dims))
    out = v.copy()
    out[..., first] = v[..., first] * c - v[..., second] * s
    out[..., second] = v[..., second] * c + v[..., first] * s
    return out


# ---------------------------------------------------------------- softmax attention
def causal_softmax(s, sink):
    """Rows of weights over the keys j <= i; ``sink`` (a score, or None) joins the denominator only."""
    T = s.shape[0]
    s = np.where(np.arange(T)[None, :] <= np.arange(T)[:, None], s, -np.inf)
    top = s.max(axis=1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    e = np.exp(s - top)
    total = e.sum(axis=1, keepdims=True)
    if sink is not None:
        total = total + np.exp(sink - top)
    return e / total


def latent_attention(h, m, t, p, eps):
    """Queries through a normed latent; keys' unrotated part and values from one normed latent per token; one rotated key
    part shared by the heads; a learned sink per head."""
    T = h.shape[0]
    H, D, Dr, Dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms_norm(h @ t[p + "dq"].T, t[p + "dq.norm"], eps) @ t[p + "uq"].T).reshape(T, H, D + Dr)
    qr = rotate(q[:, :, D:], m["rot"], True)
    low = h @ t[p + "dkv"].T
    c = rms_norm(low[:, :R], t[p + "dkv.norm"], eps)
    kr = rotate(low[:, R:], m["rot"], True)
    k = (c @ t[p + "uk"].T).reshape(T, H, D)
    v = (c @ t[p + "uv"].T).reshape(T, H, Dv)
    out = np.zeros((T, H, Dv))
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out[:, a] = causal_softmax(s, t[p + "sink"][a]) @ v[:, a]
    return out.reshape(T, H * Dv) @ t[p + "o"].T


def grouped_attention(h, m, t, p, eps):
    """Grouped-query attention: heads normed with a shared gain, then turned; capped scores; a sink of score 0; one gate per head."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ t[p + "q"].T).reshape(T, H, D), t[p + "q.norm"], eps)
    k = rms_norm((h @ t[p + "k"].T).reshape(T, G, D), t[p + "k.norm"], eps)
    v = (h @ t[p + "v"].T).reshape(T, G, Dv)
    if m.get("rot"):
        q, k = rotate(q, m["rot"], False), rotate(k, m["rot"], False)
    gate = sigmoid(h @ t[p + "g"].T)
    out = np.zeros((T, H, Dv))
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"]
        if m.get("softcap"):
            s = m["softcap"] * np.tanh(s / m["softcap"])
        out[:, a] = causal_softmax(s, 0.0) @ v[:, g] * gate[:, a:a + 1]
    return out.reshape(T, H * Dv) @ t[p + "o"].T


# ---------------------------------------------------------------- recurrences
def gated_linear_attention(h, m, t, p, eps):
    """S <- diag(alpha) S + k v^T, o = S^T q, alpha = sigmoid(W_a2 W_a1 h + b)^(1 / tau) per head and key dim."""
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ t[p + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ t[p + "k"].T).reshape(T, H, D)
    v = (h @ t[p + "v"].T).reshape(T, H, Dv)
    alpha = (sigmoid((h @ t[p + "a1"].T) @ t[p + "a2"].T + t[p + "a2.b"]) ** (1.0 / m["tau"])).reshape(T, H, D)
    S = np.zeros((H, D, Dv))
    o = np.zeros((T, H, Dv))
    for i in range(T):
        S = alpha[i][:, :, None] * S + k[i][:, :, None] * v[i][:, None, :]
        o[i] = np.einsum("hdv,hd->hv", S, q[i])
    y = rms_norm(o, t[p + "norm"], eps).reshape(T, H * Dv) * silu(h @ t[p + "g"].T)
    return y @ t[p + "o"].T


def causal_convolution(x, w, b):
    """x [T, C], w [C, taps]; the last tap belongs to the token itself, zeros before the start."""
    taps = w.shape[1]
    y = np.tile(b, (x.shape[0], 1))
    for j in range(taps):
        back = taps - 1 - j
        for i in range(back, x.shape[0]):
            y[i] += x[i - back] * w[:, j]
    return y


def state_space(h, m, t, p, eps):
    """S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x per head, behind a short convolution of x, B and C; a gate, then a
    norm in equal parts."""
    T = h.shape[0]
    H, Dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * Dv
    proj = h @ t[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_convolution(xbc, t[p + "conv"], t[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, Dv)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + t[p + "dt_bias"])
    decay = np.exp(-np.exp(t[p + "A_log"]) * dt)
    S = np.zeros((H, N, Dv))
    y = np.zeros((T, H, Dv))
    for i in range(T):
        for a in range(H):
            g = a // (H // G)
            S[a] = decay[i, a] * S[a] + dt[i, a] * np.outer(B[i, g], x[i, a])
            y[i, a] = S[a].T @ C[i, g] + t[p + "D"][a] * x[i, a]
    y = (y.reshape(T, inner) * silu(z)).reshape(T, m["norm_groups"], -1)
    y = y / np.sqrt((y * y).mean(axis=-1, keepdims=True) + eps)
    return (y.reshape(T, inner) * t[p + "norm"]) @ t[p + "o"].T


def side_by_side(h, m, t, p, eps):
    return (m["left_scale"] * grouped_attention(h, m["left"], t, p + "left.", eps)
            + m["right_scale"] * state_space(h, m["right"], t, p + "right.", eps))


MIXERS = {"gla": gated_linear_attention, "latent_attention": latent_attention, "parallel": side_by_side}


# ---------------------------------------------------------------- feed-forward
def clamped_ff(h, f, t, p):
    g = np.minimum(h @ t[p + "gate"].T, f["limit"])
    u = np.clip(h @ t[p + "up"].T, -f["limit"], f["limit"])
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ t[p + "down"].T


# ---------------------------------------------------------------- a layer, the model
def layer(x, t, l, spec, eps):
    p = f"l{l}."
    x = x + layer_norm(MIXERS[spec["type"]](x, spec["mixer"], t, p + "mix.", eps), t[p + "norm1"], t[p + "norm1.b"], eps)
    if spec.get("mlp"):
        x = x + layer_norm(clamped_ff(x, spec["mlp"], t, p + "mlp."), t[p + "norm2"], t[p + "norm2.b"], eps)
    return x


def forward(config, tensors, tokens, layer_outputs=None):
    """Logits [T, vocab] of one sequence; ``layer_outputs`` (a list) receives the stream after every layer."""
    t = {k: np.asarray(v, dtype=np.float64) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = t["embed"][np.asarray(tokens)]
    for l, spec in enumerate(config["layers"]):
        x = layer(x, t, l, spec, eps)
        if layer_outputs is not None:
            layer_outputs.append(x)
    return layer_norm(x, t["final.norm"], t["final.norm.b"], eps) @ t["head"].T
