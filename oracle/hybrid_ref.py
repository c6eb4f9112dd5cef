"""Plain numpy reference of the layer-list models (Gufanex): one function per mechanism, one sequence at a time,
every token's value written out from its equation.  float64 by default.  Shares no code with the product path:
it takes a dict name -> ndarray and the parsed configuration.

Notation: h [T, width] is a mixer's / feed-forward's input, position t counts from 0 in the sequence.
"""
from __future__ import annotations

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


MIXERS = {"mamba1": lambda W, p, m, h, eps: mamba1(W, p, m, h), "latent_attention": latent_attention}


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


def layer(W, i, entry, x, eps):
    p = f"l{i}"
    d = MIXERS[entry["type"]](W, p + ".mix", entry["mixer"], layer_norm(x, W[p + ".norm1"], W[p + ".norm1.b"], eps), eps)
    if entry.get("mlp"):
        d = d + moe(W, p + ".mlp", entry["mlp"], layer_norm(x, W[p + ".norm2"], W[p + ".norm2.b"], eps))
    return x + d


def schedule(cfg):
    """[(layer, pass or None)]: a looped layer once per pass; the first layer of a pass carries its number."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, None) for i in range(lp["stop"], n)]


def forward(W, cfg, tokens, dtype=np.float64, residuals=None):
    """Logits [T, vocab] of one sequence; residuals: a list that receives x after every layer run."""
    W = {k: np.asarray(v, dtype) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x0 = W["embed"][np.asarray(tokens)]
    x = x0
    for i, t in schedule(cfg):
        if t is not None:
            if t > 0:
                x = x + x0
            x = x + W["loop.step"][t]
        x = layer(W, i, cfg["layers"][i], x, eps)
        if residuals is not None:
            residuals.append(x)
    z = layer_norm(x, W["final.norm"], W["final.norm.b"], eps) @ W["head"].T
    cap = cfg.get("logit_softcap")
    return cap * np.tanh(z / cap) if cap else z
