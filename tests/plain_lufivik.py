"""A plain, slow implementation of the Lufivik design in float64 numpy, one function per mechanism.

Everything is written from the design's equations and shares no code with the package: whole
sequences at once, no cache, no batching.  ``forward`` takes a config.json dictionary and the
tensors by their file names.

Notation: ``x`` [T, W] the residual stream of one sequence, ``h`` a sublayer's (normed) input, ``eps`` the
norms' constant, ``t`` the tensors by file name, ``p`` the prefix of a mixer's or feed-forward's tensors,
``m`` the mixer's (or feed-forward's) object of config.json.  Linear weights are ``[out, in]`` and applied
as ``h @ W.T``.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def layer_norm(x, w, b, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


# ---------------------------------------------------------------- embedding
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Per token the row of the bigram table: (previous * mul_prev + current * mul_cur) mod buckets; the extra row
    behind the buckets for the sequence's first token."""
    out = [buckets]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        out.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return out[:len(tokens)]


def embed(tokens, config, t):
    x = t["embed"][np.asarray(tokens)]
    b = (config.get("embedding") or {}).get("bigram")
    if b:
        x = x + t["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])]
    return layer_norm(x, t["embed.norm"], t["embed.norm.b"], config["norm"]["eps"])


# ---------------------------------------------------------------- the input convolution
def causal_convolution(h, w):
    """h [T, C], w [C, taps]; the last tap belongs to the token itself, zeros before the start."""
    taps = w.shape[1]
    y = np.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        for i in range(back, h.shape[0]):
            y[i] += h[i - back] * w[:, j]
    return y


# ---------------------------------------------------------------- attention
def window_mask(T, size):
    """[i, j] true where query i sees key j: 0 <= i - j < size (``size`` None: every earlier key)."""
    back = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (back >= 0) & (back < (T if size is None else size))


def rotate(v, positions, base, dims):
    """The first ``dims`` of the last axis of v [T, ..., D] turned by position, dimension i with i + dims / 2."""
    half = dims // 2
    f = np.array([float(base) ** (-2.0 * i / dims) for i in range(half)])
    a = np.asarray(positions, dtype=np.float64)[:, None] * f                      # [T, half]
    a = a.reshape(a.shape[0], *([1] * (v.ndim - 2)), half)
    u, w = v[..., :half], v[..., half:dims]
    return np.concatenate([u * np.cos(a) - w * np.sin(a), w * np.cos(a) + u * np.sin(a), v[..., dims:]], axis=-1)


def latent_attention(h, m, t, p, eps):
    """Every head's unrotated keys and its values come from one normed latent per token; one rotated key part is
    shared by the heads; a window; a sigmoid gate per head."""
    T = h.shape[0]
    H, D, Dr, Dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    pos = np.arange(T)
    cq = rms_norm(h @ t[p + "dq"].T, t[p + "dq.norm"], eps)
    q = (cq @ t[p + "uq"].T).reshape(T, H, D + Dr)
    qr = rotate(q[:, :, D:], pos, base, dims)
    low = h @ t[p + "dkv"].T
    c = rms_norm(low[:, :R], t[p + "dkv.norm"], eps)
    kr = rotate(low[:, R:], pos, base, dims)                                      # [T, Dr]
    k = (c @ t[p + "uk"].T).reshape(T, H, D)
    v = (c @ t[p + "uv"].T).reshape(T, H, Dv)
    mask = window_mask(T, (m.get("mask") or {}).get("size"))
    gate = sigmoid(h @ t[p + "g"].T)
    out = np.zeros((T, H, Dv))
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        s = np.where(mask, s, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, a] = (e / e.sum(axis=1, keepdims=True)) @ v[:, a] * gate[:, a:a + 1]
    return out.reshape(T, H * Dv) @ t[p + "o"].T


# ---------------------------------------------------------------- feed-forward
def expert(h, t, p, limit):
    g = np.minimum(h @ t[p + "gate"].T, limit)
    u = np.clip(h @ t[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ t[p + "down"].T


def route(z, top):
    """Chosen experts [T, top] (largest scores, the lower index among equals) and their softmax scores."""
    e = np.exp(z - z.max(axis=1, keepdims=True))
    s = e / e.sum(axis=1, keepdims=True)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


def experts_ff(h, f, t, p):
    chosen, w = route(h @ t[p + "router"].T, f["router"]["top"])
    out = np.zeros((h.shape[0], t[p + "e0.down"].shape[0]))
    for e in range(f["router"]["experts"]):
        rows, ranks = np.nonzero(chosen == e)
        if len(rows):
            out[rows] += w[rows, ranks][:, None] * expert(h[rows], t, f"{p}e{e}.", f["expert"]["limit"])
    return out


# ---------------------------------------------------------------- a layer, the order of layers, the model
def sublayer(x, t, l, n, eps, run, canon=False):
    """x + ls * norm_out(sigmoid(W h + b) * run(h')), h = norm_in(x), h' = h (+ conv(h))."""
    p = f"l{l}."
    h = layer_norm(x, t[f"{p}norm{n}"], t[f"{p}norm{n}.b"], eps)
    y = run(h + causal_convolution(h, t[f"{p}canon1"]) if canon else h)
    y = y * sigmoid(h @ t[f"{p}rg{n}"].T + t[f"{p}rg{n}.b"])
    return x + t[f"{p}ls{n}"] * layer_norm(y, t[f"{p}norm{n}b"], t[f"{p}norm{n}b.b"], eps)


def layer(x, t, l, spec, eps):
    x = sublayer(x, t, l, 1, eps, lambda h: latent_attention(h, spec["mixer"], t, f"l{l}.mix.", eps), canon=True)
    if spec.get("mlp"):
        x = sublayer(x, t, l, 2, eps, lambda h: experts_ff(h, spec["mlp"], t, f"l{l}.mlp."))
    return x


def run_order(config):
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


def forward(config, tensors, tokens, layer_outputs=None):
    """Logits [T, vocab] of one sequence; ``layer_outputs`` (a list) receives the stream after every layer run."""
    t = {k: np.asarray(v, dtype=np.float64) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = embed(tokens, config, t)
    for l in run_order(config):
        x = layer(x, t, l, config["layers"][l], eps)
        if layer_outputs is not None:
            layer_outputs.append(x)
    return layer_norm(x, t["final.norm"], t["final.norm.b"], eps) @ t["head"].T
