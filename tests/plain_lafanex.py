"""A plain, slow Lafanex: whole sequences, no cache, no carried state, float64, one function a mechanism.

It shares no code with `liyab_amd`: it takes a dict of numpy tensors by their file names and config.json
as a dict, and computes with numpy from the design's equations. In this file's notation (rows = tokens; p: a row's
position; unit(v) = v / sqrt(mean(v^2) + eps); n(v) = unit(v) (1 + w); s: the logistic function):

  X       = S copies of embed[token]                                   (S = config's streams; one plain stream without that key)
  sublayer q of a layer (1: mixer, 2: feed-forward), with a (in), M (mix, [from, to]) and b (out):
            y = f_q(n_q(a X));  X <- M^T X + b y                        (plain stream: x <- x + f_q(n_q(x)))
  logits  = embed n_f(sum of X)
  config's loop: layers start .. stop - 1 run `times` times in a row, then the rest

  mixer "attention": q, k, v = W h; the first rot.dims entries of every head in pairs (2i, 2i + 1) turned by p base^(-2i / dims);
      unit over a head of q and of k; row i sees rows j <= i; weights exp(scale q.k) / (1 + sum of exp); Wo.
  mixer "mamba1":    [x | z] = Win h; x <- silu(conv(x) + b) over time, a channel each; [d | B | C] = Wx x; d <- softplus(Wdt d + b);
      S[c, n] <- exp(-d_c exp(A_log[c, n])) S[c, n] + d_c x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c;  Wo (y silu(z)).
  feed-forward "dense": Wd (gelu(Wg h) * (Wu h))
  feed-forward "moe":   p = softmax(Wr h) over experts and identity outputs; the `top` largest p + correction, weighted scale p;
      expert: g = min(Wg h, limit), u = clamp(Wu h, -limit, limit), Wd (g s(1.702 g) (u + 1)); identity: h itself;
      one more such expert for every token times s(Wsg h).
"""

from __future__ import annotations

import math

import numpy as np


def round_to_bf16(a):
    """float -> the nearest bfloat16 (ties to even), as float64."""
    f = np.ascontiguousarray(a, dtype=np.float32)
    bits = f.view(np.uint32).astype(np.uint64)
    bits = (bits + 0x7FFF + ((bits >> 16) & 1)) & 0xFFFF0000
    return bits.astype(np.uint32).view(np.float32).astype(np.float64).reshape(np.shape(a))


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def silu(z):
    return z * logistic(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def unit(v, eps):
    """v / sqrt(mean(v^2) + eps) over the last axis."""
    return v / np.sqrt((v * v).mean(axis=-1, keepdims=True) + eps)


def stored_norm(v, w, eps):
    return unit(v, eps) * (1.0 + w)


def turn_pairs(v, positions, rot):
    """v [n, heads, dim]: pairs (2i, 2i + 1) of the first rot.dims entries turned by position * base^(-2i / dims)."""
    dims = rot["dims"]
    f = np.array([rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)])
    a = positions[:, None] * f[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    out = v.copy()
    even, odd = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = even * c - odd * s
    out[..., 1:dims:2] = odd * c + even * s
    return out


def weights_with_one(scores, seen):
    """exp(s_j) / (1 + sum of exp(s)) over the rows that are seen."""
    s = np.where(seen, scores, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    p = np.exp(s - m)
    return p / (np.exp(-m) + p.sum(axis=-1, keepdims=True))


def attention(h, t, prefix, m, positions, eps):
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ t[prefix + "q"].T).reshape(n, H, D)
    k = (h @ t[prefix + "k"].T).reshape(n, G, D)
    v = (h @ t[prefix + "v"].T).reshape(n, G, V)
    if m.get("rot"):
        q, k = turn_pairs(q, positions, m["rot"]), turn_pairs(k, positions, m["rot"])
    q, k = unit(q, eps), unit(k, eps)
    seen = np.arange(n)[None, :] <= np.arange(n)[:, None]
    out = np.zeros((n, H, V))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = weights_with_one((q[:, hd] @ k[:, g].T) * m["scale"], seen) @ v[:, g]
    return out.reshape(n, -1) @ t[prefix + "o"].T


def short_convolution(x, w, b):
    """x [n, channels], w [channels, taps] (last column: the current row), zeros before the first row."""
    n, taps = x.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    out = np.zeros_like(x) + b
    for j in range(taps):
        out += w[:, j] * padded[j:j + n]
    return out


def selective_walk(x, d, B, C, A, skip):
    """x, d [n, channels], B, C [n, states], A [channels, states] -> y [n, channels]."""
    S = np.zeros(A.shape)
    y = np.zeros_like(x)
    for i in range(x.shape[0]):
        S = np.exp(d[i][:, None] * A) * S + (d[i] * x[i])[:, None] * B[i][None, :]
        y[i] = S @ C[i] + skip * x[i]
    return y


def mamba1(h, t, prefix, m):
    inner, rank, N = m["inner"], m["dt_rank"], m["state"]
    xz = h @ t[prefix + "in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(short_convolution(x, t[prefix + "conv"], t[prefix + "conv.b"]))
    dbc = x @ t[prefix + "x"].T
    d = softplus(dbc[:, :rank] @ t[prefix + "dt"].T + t[prefix + "dt.b"])
    y = selective_walk(x, d, dbc[:, rank:rank + N], dbc[:, rank + N:], -np.exp(t[prefix + "A_log"]), t[prefix + "D"])
    return (y * silu(z)) @ t[prefix + "o"].T


def clamped_unit(h, t, prefix, limit):
    g = np.minimum(h @ t[prefix + "gate"].T, limit)
    u = np.clip(h @ t[prefix + "up"].T, -limit, limit)
    return (g * logistic(1.702 * g) * (u + 1.0)) @ t[prefix + "down"].T


def route(z, correction, top, scale):
    """z [n, outputs] router logits -> (chosen [n, top], weights [n, top])."""
    p = np.exp(z - z.max(axis=-1, keepdims=True))
    p = p / p.sum(axis=-1, keepdims=True)
    chosen = np.argsort(-(p + correction), axis=-1, kind="stable")[:, :top]
    return chosen, scale * np.take_along_axis(p, chosen, axis=-1)


def routed_feed_forward(h, t, prefix, m, router_input=None):
    r = m["router"]
    chosen, weights = route((h if router_input is None else router_input) @ t[prefix + "router"].T, t[prefix + "correction"], r["top"], r.get("scale", 1.0))
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        for e, w in zip(chosen[i], weights[i]):
            out[i] += w * (h[i] if e >= r["experts"] else clamped_unit(h[i:i + 1], t, f"{prefix}e{e}.", m["expert"]["limit"])[0])
    if m.get("shared"):
        out += logistic(h @ t[prefix + "shared.sg"].T) * clamped_unit(h, t, prefix + "shared.", m["shared"]["limit"])
    return out


def feed_forward(h, t, prefix, m):
    if m["kind"] == "dense":
        return (gelu_tanh(h @ t[prefix + "gate"].T) * (h @ t[prefix + "up"].T)) @ t[prefix + "down"].T
    return routed_feed_forward(h, t, prefix, m)


def connected(X, t, prefix, sublayer):
    """X [streams, n, width] -> the streams behind the sublayer; the sums by entries of the three tensors."""
    a, b, M = t[prefix + "in"], t[prefix + "out"], t[prefix + "mix"]
    S = X.shape[0]
    y = sublayer(sum(a[s] * X[s] for s in range(S)))
    return np.stack([sum(M[s, to] * X[s] for s in range(S)) + b[to] * y for to in range(S)])


def runs(config):
    loop = config.get("loop")
    n = len(config["layers"])
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + loop["times"] * list(range(loop["start"], loop["stop"])) + list(range(loop["stop"], n))


def forward(config, t, tokens, streams=None):
    """float64 logits [n, vocab] of a whole sequence; `streams` (a list) gets the streams' sum after every run of a layer."""
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens), dtype=np.float64)
    eps = config["norm"]["eps"]
    S = config.get("streams")
    X = np.stack([t["embed"][tokens].astype(np.float64)] * (S or 1))
    for i in runs(config):
        layer = config["layers"][i]
        p, m = f"l{i}.", layer["mixer"]

        def mix(x):
            h = stored_norm(x, t[p + "norm1"], eps)
            if layer["type"] == "attention":
                return attention(h, t, p + "mix.", m, positions, eps)
            if layer["type"] == "mamba1":
                return mamba1(h, t, p + "mix.", m)
            raise ValueError(layer["type"])

        def feed(x):
            return feed_forward(stored_norm(x, t[p + "norm2"], eps), t, p + "mlp.", layer["mlp"])

        for q, sublayer in ((1, mix), (2, feed if layer.get("mlp") else None)):
            if sublayer is None:
                continue
            X = connected(X, t, f"{p}hc{q}.", sublayer) if S else X + sublayer(X[0])
        if streams is not None:
            streams.append(X.sum(axis=0))
    return stored_norm(X.sum(axis=0), t["final.norm"], eps) @ t["embed"].T
