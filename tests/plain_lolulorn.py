"""A plain, slow Lolulorn: whole sequences, no cache, no carried state, float64, one function a mechanism.

It shares no code with `liyab_amd`: it takes a dict of numpy tensors by their file names and config.json
as a dict, and computes with numpy from the design's equations. In this file's notation (x: the residual
stream, rows = tokens; p: a row's position; unit(v) = v / sqrt(mean(v^2) + eps); N(v) = (v - mean) /
sqrt(var + eps) w + b; s: the logistic function):

  x_0     = scale * embed[token]
  layer:    x <- x + N1(mixer(x));  x <- x + N2(ff(x))                 (a layer may have no feed-forward)
  logits  = head N_f(x)

  mixer "attention": q, k, v = W x; unit over all of q's (and k's) entries at once, a weight an entry; the first
      rot.dims entries of every head in pairs (2i, 2i + 1) turned by p base^(-2i / dims) / factor; row i sees row j <= i if
      i - j < size or j < keep_first; softmax(scale q.k); Wo. A layer with kv_from takes the keys and values of that layer.
  mixer "delta":     q, k, v = silu(conv(W x)) over time, a channel each; q and k of every head to length one, q times
      dim^(-1/2); r = s(Wb x), g = exp(-exp(A_log) softplus(Wa x + dt_bias)); S <- g S; S <- S + k (r (v - S^T k))^T; o = S^T q;
      unit over a head's o, a weight, times silu(Wg x); Wo. Heads share q and k in groups.
  mixer "gla":       q = Wq x dim^(-1/2), k, v = W x; a = s(Wa2 (Wa1 x) + b)^(1 / tau) an entry of k; S <- diag(a) S + k v^T;
      o = S^T q; unit over a head's o, a weight, times silu(Wg x); Wo.
  feed-forward "dense": Wd (gelu(Wg x) * (Wu x))
  feed-forward "moe":   c = s(Wr x) + correction; experts in groups.count groups of neighbours, a group's score the sum of
      its two largest c, the best groups.keep groups stay; of their experts the `top` largest c, weighted by s(Wr x);
      sum of weight * Wd (silu(Wg x) * (Wu x)).
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


def centred_norm(v, w, b, eps):
    c = v - v.mean(axis=-1, keepdims=True)
    return c / np.sqrt((c * c).mean(axis=-1, keepdims=True) + eps) * w + b


def turn_pairs(v, positions, rot):
    """v [n, heads, dim]: pairs (2i, 2i + 1) of the first rot.dims entries turned by position * f_i."""
    dims = rot["dims"]
    f = np.array([rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)])
    if rot.get("scaling"):
        f = f / rot["scaling"]["factor"]
    a = positions[:, None] * f[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    out = v.copy()
    even, odd = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = even * c - odd * s
    out[..., 1:dims:2] = odd * c + even * s
    return out


def visible(n, mask):
    """[n, n]: whether row i sees row j."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < mask["size"]) | (j < mask["keep_first"]))
    return seen


def softmax_over(scores, seen):
    s = np.where(seen, scores, -np.inf)
    p = np.exp(s - s.max(axis=-1, keepdims=True))
    return p / p.sum(axis=-1, keepdims=True)


def keys_and_values(h, t, prefix, m, positions, eps):
    n, G = h.shape[0], m["kv_heads"]
    k = (unit(h @ t[prefix + "k"].T, eps) * t[prefix + "k.norm"]).reshape(n, G, m["dim"])
    if m.get("rot"):
        k = turn_pairs(k, positions, m["rot"])
    return k, (h @ t[prefix + "v"].T).reshape(n, G, m["vdim"])


def attention(h, t, prefix, m, positions, eps, kv):
    """kv: the keys [n, G, dim] and values [n, G, vdim] that the layer's queries meet."""
    n, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (unit(h @ t[prefix + "q"].T, eps) * t[prefix + "q.norm"]).reshape(n, H, D)
    if m.get("rot"):
        q = turn_pairs(q, positions, m["rot"])
    k, v = kv
    seen = visible(n, m.get("mask"))
    out = np.zeros((n, H, m["vdim"]))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = softmax_over((q[:, hd] @ k[:, g].T) * m["scale"], seen) @ v[:, g]
    return out.reshape(n, -1) @ t[prefix + "o"].T


def short_convolution(x, w):
    """x [n, channels], w [channels, taps] (last column: the current row), zeros before the first row."""
    n, taps = x.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    out = np.zeros_like(x)
    for j in range(taps):
        out += w[:, j] * padded[j:j + n]
    return out


def finish_heads(o, h, t, prefix, eps):
    """o [n, H, vdim] -> the mixer's result: unit a head, a weight, the gate, the output matrix."""
    n = o.shape[0]
    return ((unit(o, eps) * t[prefix + "norm"]).reshape(n, -1) * silu(h @ t[prefix + "g"].T)) @ t[prefix + "o"].T


def delta(h, t, prefix, m, eps):
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_convolution(h @ t[prefix + c].T, t[prefix + c + ".conv"])) for c in "qkv")
    q, k, v = q.reshape(n, G, D), k.reshape(n, G, D), v.reshape(n, H, V)
    q = q / np.sqrt((q * q).sum(axis=-1, keepdims=True) + 1e-6) * D ** -0.5
    k = k / np.sqrt((k * k).sum(axis=-1, keepdims=True) + 1e-6)
    rate = logistic(h @ t[prefix + "b"].T)
    decay = np.exp(-np.exp(t[prefix + "A_log"]) * softplus(h @ t[prefix + "a"].T + t[prefix + "dt_bias"]))
    o = np.zeros((n, H, V))
    for hd in range(H):
        g = hd // (H // G)
        S = np.zeros((D, V))
        for i in range(n):
            S = decay[i, hd] * S
            S = S + np.outer(k[i, g], rate[i, hd] * (v[i, hd] - S.T @ k[i, g]))
            o[i, hd] = S.T @ q[i, g]
    return finish_heads(o, h, t, prefix, eps)


def gla(h, t, prefix, m, eps):
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ t[prefix + "q"].T).reshape(n, H, D) * D ** -0.5
    k = (h @ t[prefix + "k"].T).reshape(n, H, D)
    v = (h @ t[prefix + "v"].T).reshape(n, H, V)
    z = (h @ t[prefix + "a1"].T) @ t[prefix + "a2"].T + t[prefix + "a2.b"]
    a = np.exp(-softplus(-z) / m["tau"]).reshape(n, H, D)  # s(z)^(1 / tau)
    o = np.zeros((n, H, V))
    for hd in range(H):
        S = np.zeros((D, V))
        for i in range(n):
            S = a[i, hd][:, None] * S + np.outer(k[i, hd], v[i, hd])
            o[i, hd] = S.T @ q[i, hd]
    return finish_heads(o, h, t, prefix, eps)


def gated_unit(h, t, prefix, act):
    return (act(h @ t[prefix + "gate"].T) * (h @ t[prefix + "up"].T)) @ t[prefix + "down"].T


def route(z, correction, top, groups, keep):
    """z [n, E] router logits -> (chosen [n, top], weights [n, top])."""
    n, E = z.shape
    s = logistic(z)
    c = s + correction
    per = E // groups
    chosen, weights = np.zeros((n, top), dtype=np.int64), np.zeros((n, top))
    for i in range(n):
        score = np.sort(c[i].reshape(groups, per), axis=-1)[:, -2:].sum(axis=-1)
        best = np.argsort(-score, kind="stable")[:keep]
        allowed = np.full(E, -np.inf)
        for g in best:
            allowed[g * per:(g + 1) * per] = c[i, g * per:(g + 1) * per]
        chosen[i] = np.argsort(-allowed, kind="stable")[:top]
        weights[i] = s[i, chosen[i]]
    return chosen, weights


def routed_feed_forward(h, t, prefix, m, router_input=None):
    r = m["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = (h if router_input is None else router_input) @ t[prefix + "router"].T
    chosen, weights = route(z, t[prefix + "correction"], r["top"], groups["count"], groups["keep"])
    out = np.zeros((h.shape[0], t[prefix + "e0.down"].shape[0]))
    for i in range(h.shape[0]):
        for e, w in zip(chosen[i], weights[i]):
            out[i] += w * gated_unit(h[i:i + 1], t, f"{prefix}e{e}.", silu)[0]
    return out


def feed_forward(h, t, prefix, m):
    if m["kind"] == "dense":
        return gated_unit(h, t, prefix, gelu_tanh)
    return routed_feed_forward(h, t, prefix, m)


def forward(config, t, tokens, streams=None):
    """float64 logits [n, vocab] of a whole sequence; `streams` (a list) gets the stream after every layer."""
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens), dtype=np.float64)
    eps = config["norm"]["eps"]
    x = t["embed"][tokens].astype(np.float64) * config["embedding"]["scale"]
    kept = {}  # keys and values by layer

    def norm(v, name):
        return centred_norm(v, t[name], t[name + ".b"], eps)

    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        if layer["type"] == "attention":
            if m.get("kv_from") is None:
                kept[i] = keys_and_values(x, t, p + "mix.", m, positions, eps)
            y = attention(x, t, p + "mix.", m, positions, eps, kept[i if m.get("kv_from") is None else m["kv_from"]])
        elif layer["type"] == "delta":
            y = delta(x, t, p + "mix.", m, eps)
        elif layer["type"] == "gla":
            y = gla(x, t, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + norm(y, p + "norm1")
        if layer.get("mlp") is not None:
            x = x + norm(feed_forward(x, t, p + "mlp.", layer["mlp"]), p + "norm2")
        if streams is not None:
            streams.append(x.copy())
    return norm(x, "final.norm") @ t["head"].T
