"""Plain numpy reference of the layer-list models (Gufanex, Gusorax): one function per mechanism, one sequence at a time,
every token's value written out from its equation.  float64 by default.  Shares no code with the product path:
it takes a dict name -> ndarray and the parsed configuration.

Notation: h [T, width] is a mixer's / feed-forward's input, position t counts from 0 in the sequence.
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


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def layer_norm(x, w, b, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w + b


def causal_conv(x, w, b):
    """Depthwise convolution: y[t, c] = b_c + sum_k w[c, k] x[t - (taps-1) + k, c], zeros before the start."""
    taps = w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, x.shape[1]), x.dtype), x])
    y = np.zeros_like(x) + b
    for k in range(taps):
        y = y + pad[k: k + len(x)] * w[:, k]
    return y


def selective_scan(x, dt, A, B, C, D):
    """S_t = exp(dt_t A) S_{t-1} + (dt_t x_t) B_t ;  y_t = S_t . C_t + D x_t ;  S_{-1} = 0.  x, dt [T, c]; A [c, n];
    B, C [T, n]."""
    S = np.zeros_like(A)
    y = np.zeros_like(x)
    for t in range(len(x)):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba1(W, p, m, h):
    """W: tensors, p: prefix '<layer>.mix', m: the mixer's sizes."""
    inner, n, r = m["inner"], m["state"], m["dt_rank"]
    xz = h @ W[p + ".in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, W[p + ".conv"], W[p + ".conv.b"]))
    dbc = x @ W[p + ".x"].T
    dt = softplus(dbc[:, :r] @ W[p + ".dt"].T + W[p + ".dt.b"])
    y = selective_scan(x, dt, -np.exp(W[p + ".A_log"]), dbc[:, r: r + n], dbc[:, r + n:], W[p + ".D"])
    return (y * silu(z)) @ W[p + ".o"].T


def rope_interleaved(v, base, dims):
    """v [T, ..., d]: pairs (2i, 2i+1) of the first `dims` entries turn by t * base^(-2i/dims)."""
    T = v.shape[0]
    f = float(base) ** (-2.0 * np.arange(dims // 2) / dims)
    a = (np.arange(T)[:, None] * f[None, :]).reshape((T,) + (1,) * (v.ndim - 2) + (dims // 2,))
    out = v.copy()
    u, w = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = u * np.cos(a) - w * np.sin(a)
    out[..., 1:dims:2] = w * np.cos(a) + u * np.sin(a)
    return out


def softmax_sink(s, sink):
    """Rows of s [T, H, T] with the extra term exp(sink_h) in the denominator."""
    m = np.maximum(s.max(axis=-1), sink)
    e = np.exp(s - m[..., None])
    return e / (e.sum(axis=-1) + np.exp(sink - m))[..., None]


def latent_attention(W, p, m, h, eps):
    T = len(h)
    H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms_norm(h @ W[p + ".dq"].T, W[p + ".dq.norm"], eps)
    q = (cq @ W[p + ".uq"].T).reshape(T, H, dn + dr)
    kv = h @ W[p + ".dkv"].T
    c = rms_norm(kv[:, :R], W[p + ".dkv.norm"], eps)
    kr = rope_interleaved(kv[:, R:], m["rot"]["base"], m["rot"]["dims"])
    qr = rope_interleaved(q[:, :, dn:], m["rot"]["base"], m["rot"]["dims"])
    kn = (c @ W[p + ".uk"].T).reshape(T, H, dn)
    v = (c @ W[p + ".uv"].T).reshape(T, H, dv)
    s = (np.einsum("thd,jhd->thj", q[:, :, :dn], kn) + np.einsum("thd,jd->thj", qr, kr)) * m["scale"]
    t = np.arange(T)
    s = np.where(t[None, None, :] <= t[:, None, None], s, -np.inf)
    a = softmax_sink(s, W[p + ".sink"])
    return np.einsum("thj,jhv->thv", a, v).reshape(T, H * dv) @ W[p + ".o"].T


def distance_bucket(n, rows, far):
    """Row of a distance table of `rows` entries: one entry per distance below half of them, then entries of equal
    width in log distance up to `far`, the last one for everything beyond."""
    half = rows // 2
    if n < half:
        return n
    x = math.log(n / half) / math.log(far / half) * (rows - half)
    r = round(x)
    if abs(x - r) < 1e-9:  # a border up to rounding of the logarithms
        x = r
    return min(rows - 1, half + math.floor(x))


def visible(T, window=None, chunk=None):
    """[T, T] booleans: query t (row) sees key j."""
    t, j = np.arange(T)[:, None], np.arange(T)[None, :]
    v = j <= t
    if window is not None:
        v &= t - j < window
    if chunk is not None:
        v &= t // chunk == j // chunk
    return v


def heads(W, p, h, n, d):
    """Projection p of h, split into n heads; its bias if the model has one."""
    y = h @ W[p].T
    if p + ".b" in W:
        y = y + W[p + ".b"]
    return y.reshape(len(h), n, d)


def softmax_extra(s, extra):
    """Rows of s [T, H, T] over the last axis with the constant `extra` in the denominator, in units of exp(0)."""
    m = np.maximum(s.max(axis=-1), 0.0 if extra else -np.inf)
    e = np.exp(s - m[..., None])
    return e / (e.sum(axis=-1) + (extra * np.exp(-m) if extra else 0.0))[..., None]


def grouped_attention(W, p, m, h, eps, seen, bias=None, extra=0.0, gate=False):
    """Query head a uses key / value head a // (heads / kv_heads); per-head RMS norms of queries and keys; bias
    [heads, T, T] is added to the scaled scores."""
    T, H, G, dk, dv = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(heads(W, p + ".q", h, H, dk), W[p + ".q.norm"], eps)
    k = rms_norm(heads(W, p + ".k", h, G, dk), W[p + ".k.norm"], eps)
    v = heads(W, p + ".v", h, G, dv)
    out = np.zeros((T, H, dv), h.dtype)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"]
        if bias is not None:
            s = s + bias[a]
        w = softmax_extra(np.where(seen, s, -np.inf)[:, None], extra)[:, 0]
        out[:, a] = w @ v[:, g]
    out = out.reshape(T, H * dv)
    if gate:
        out = out * sigmoid(h @ W[p + ".g"].T)
    y = out @ W[p + ".o"].T
    return y + W[p + ".o.b"] if p + ".o.b" in W else y


def window_attention(W, p, m, h, eps):
    """Sliding window and a learned bias by distance."""
    T, rel = len(h), W[p + ".rel"]
    row = [distance_bucket(n, len(rel), m["bias_max"]) for n in range(T)]
    d = np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0)
    bias = rel[np.array(row)[d]].transpose(2, 0, 1)
    return grouped_attention(W, p, m, h, eps, visible(T, window=m["mask"]["size"]), bias=bias)


def chunk_attention(W, p, m, h, eps):
    """Chunks of the sequence, a sink of score 0 and an output gate."""
    return grouped_attention(W, p, m, h, eps, visible(len(h), chunk=m["mask"]["size"]), extra=1.0, gate=True)


MIXERS = {"mamba1": lambda W, p, m, h, eps: mamba1(W, p, m, h), "latent_attention": latent_attention,
          "attention": window_attention, "attention_2": chunk_attention}


def gated_mlp(W, p, h):
    return (silu(h @ W[p + ".gate"].T) * (h @ W[p + ".up"].T)) @ W[p + ".down"].T


def route(z, correction, top):
    """Scores, chosen ids [T, top] by score + correction, and the chosen experts' plain scores as weights."""
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    s = e / e.sum(axis=-1, keepdims=True)
    ids = np.argsort(-(s + correction), axis=-1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, axis=-1)


def moe(W, p, m, h):
    r = m["router"]
    ids, w = route(h @ W[p + ".router"].T, W[p + ".correction"], r["top"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, g in zip(ids[t], w[t]):
            y = gated_mlp(W, f"{p}.e{e}", h[t: t + 1])[0] if e < r["experts"] else h[t]
            out[t] += g * y
    if m.get("shared"):
        out += sigmoid(h @ W[p + ".shared.sg"].T) * gated_mlp(W, p + ".shared", h)
    return out


def clamped_expert(W, p, h, limit):
    g, u = np.minimum(h @ W[p + ".gate"].T, limit), np.clip(h @ W[p + ".up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[p + ".down"].T


def route_chosen(z, top):
    """The `top` largest outputs, weighted by the softmax over them alone."""
    ids = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    c = np.take_along_axis(z, ids, axis=-1)
    e = np.exp(c - c.max(axis=-1, keepdims=True))
    return ids, e / e.sum(axis=-1, keepdims=True)


def clamped_moe(W, p, m, h):
    ids, w = route_chosen(h @ W[p + ".router"].T, m["router"]["top"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, g in zip(ids[t], w[t]):
            out[t] += g * clamped_expert(W, f"{p}.e{e}", h[t: t + 1], m["expert"]["limit"])[0]
    return out


def feed_forward(W, p, m, h):
    return gated_mlp(W, p, h) if m["kind"] == "dense" else clamped_moe(W, p, m, h)


def schedule(cfg):
    """[(layer, pass or None)]: a looped layer once per pass; the first layer of a pass carries its number."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, None) for i in range(lp["stop"], n)]


class Gufanex:
    """Two layer norms around a parallel block; a pass of the loop adds the embedding output and a step vector."""
    embed = staticmethod(lambda W, cfg, tokens: W["embed"][tokens])

    @staticmethod
    def enter(W, x, x0, t):
        return (x + x0 if t > 0 else x) + W["loop.step"][t]

    @staticmethod
    def layer(W, i, cfg, x):
        p, entry, eps = f"l{i}", cfg["layers"][i], cfg["norm"]["eps"]
        d = MIXERS[entry["type"]](W, p + ".mix", entry["mixer"], layer_norm(x, W[p + ".norm1"], W[p + ".norm1.b"], eps), eps)
        if entry.get("mlp"):
            d = d + moe(W, p + ".mlp", entry["mlp"], layer_norm(x, W[p + ".norm2"], W[p + ".norm2.b"], eps))
        return x + d

    @staticmethod
    def final(W, cfg, x):
        z = layer_norm(x, W["final.norm"], W["final.norm.b"], cfg["norm"]["eps"]) @ W["head"].T
        cap = cfg.get("logit_softcap")
        return cap * np.tanh(z / cap) if cap else z


class Gusorax:
    """One RMS norm (weights around zero) in front of a parallel block; scaled embeddings with learned positions; a pass
    of the loop enters through a matrix over [x; embedding output]."""
    @staticmethod
    def embed(W, cfg, tokens):
        return W["embed"][tokens] * cfg["embedding"]["scale"] + W["pos"][: len(tokens)]

    @staticmethod
    def enter(W, x, x0, t):
        return np.concatenate([x, x0], axis=-1) @ W["loop.in"].T

    @staticmethod
    def layer(W, i, cfg, x):
        p, entry, eps = f"l{i}", cfg["layers"][i], cfg["norm"]["eps"]
        h = rms_norm(x, 1.0 + W[p + ".norm1"], eps)
        d = MIXERS[entry["type"]](W, p + ".mix", entry["mixer"], h, eps)
        if entry.get("mlp"):
            d = d + feed_forward(W, p + ".mlp", entry["mlp"], h)
        return x + cfg["residual_mult"] * d

    @staticmethod
    def final(W, cfg, x):
        return rms_norm(x, 1.0 + W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T


ARCHITECTURES = {"Gufanex": Gufanex, "Gusorax": Gusorax}


def forward(W, cfg, tokens, dtype=np.float64, residuals=None):
    """Logits [T, vocab] of one sequence; residuals: a list that receives x after every layer run."""
    W = {k: np.asarray(v, dtype) for k, v in W.items()}
    A = ARCHITECTURES[cfg["architecture"]]
    x = x0 = A.embed(W, cfg, np.asarray(tokens))
    for i, t in schedule(cfg):
        if t is not None:
            x = A.enter(W, x, x0, t)
        x = A.layer(W, i, cfg, x)
        if residuals is not None:
            residuals.append(x)
    return A.final(W, cfg, x)
