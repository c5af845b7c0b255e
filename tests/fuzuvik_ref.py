"""Plain float64 implementation of the Fuzuvik decoder, one function per
mechanism, written from the equations.  It shares no code with the product and
is slow on purpose: attention walks queries one by one over full score rows,
recurrences walk tokens one by one, and nothing is cached.

A model is (cfg, w): cfg the decoded config.json, w a dict name -> array."""
import math

import numpy as np

UNIT_EPS = 1e-6  # inside the root of the unit vectors of the delta rule


def rms(x, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.asarray(z, np.float64)))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu(z):
    return 0.5 * z * (1.0 + np.vectorize(math.erf)(z / math.sqrt(2.0)))


def frequencies(rot):
    """One frequency per rotated pair; long wavelengths slowed down by a factor,
    with a ramp between the two regions."""
    n = rot["dims"]
    sc = rot.get("scaling")
    out = []
    for i in range(n // 2):
        f = rot["base"] ** (-2.0 * i / n)
        if sc:
            wave = 2.0 * math.pi / f
            short, long = sc["original"] / sc["high"], sc["original"] / sc["low"]
            if wave > long:
                f = f / sc["factor"]
            elif wave >= short:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate(x, p, freqs):
    """x [.., dim] at position p: the halves of the first 2 * len(freqs) values are pairs"""
    n = len(freqs)
    y = np.array(x, np.float64)
    c, s = np.cos(p * freqs), np.sin(p * freqs)
    u, v = np.array(y[..., :n]), np.array(y[..., n:2 * n])
    y[..., :n] = u * c - v * s
    y[..., n:2 * n] = v * c + u * s
    return y


def sink_softmax(s):
    """weights of scores beside a sink of score 0 that has no value"""
    top = max(0.0, float(np.max(s)))
    e = np.exp(s - top)
    return e / (math.exp(-top) + e.sum())


def chunked_attention(q, k, v, scale, size):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; a position sees itself and
    what came before it in its own chunk (size 0: everything before it)"""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        lo = i // size * size if size else 0
        for h in range(H):
            out[i, h] = sink_softmax(k[lo:i + 1, h // rep] @ q[i, h] * scale) @ v[lo:i + 1, h // rep]
    return out


def attention(h, get, m, eps, first):
    """first: a list that receives the values of the first layer that mixes values"""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = (h @ get("q").T).reshape(T, H, d), (h @ get("k").T).reshape(T, G, d)
    v = (h @ get("v").T).reshape(T, G, e)
    if m.get("rot"):
        f = frequencies(m["rot"])
        q = np.stack([rotate(q[p], p, f) for p in range(T)])
        k = np.stack([rotate(k[p], p, f) for p in range(T)])
    q, k = rms(q, eps), rms(k, eps)
    if m.get("v_mix"):
        if first:
            lam = float(get("vmix"))
            v = (1.0 - lam) * v + lam * first[0]
        else:
            first.append(v)
    size = m["mask"]["size"] if m.get("mask") else 0
    return chunked_attention(q, k, v, m["scale"], size).reshape(T, -1) @ get("o").T


def short_conv(x, w):
    """x [T, n], w [n, taps], the last column meets the current row"""
    taps = w.shape[1]
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            at = t - (taps - 1 - j)
            if at >= 0:
                y[t] += w[:, j] * x[at]
    return y


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, e], g [T, H, d] decays, beta [T, H] -> [T, H, e]"""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros(v.shape)
    for t in range(T):
        for h in range(H):
            S[h] *= g[t, h][:, None]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] += np.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out


def channel_delta(h, get, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    parts = {n: silu(short_conv(h @ get(n).T, get(n + ".conv"))) for n in "qkv"}
    q, k, v = parts["q"].reshape(T, G, d), parts["k"].reshape(T, G, d), parts["v"].reshape(T, H, e)
    q, k = (x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + UNIT_EPS) for x in (q, k))
    q = q * d ** -0.5
    q, k = np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1)
    beta = sigmoid(h @ get("b").T)
    z = (h @ get("a1").T) @ get("a2").T + get("dt_bias")
    g = np.exp(-np.exp(get("A_log"))[None, :, None] * softplus(z).reshape(T, H, d))
    o = rms(delta_rule(q, k, v, g, beta), eps) * get("norm")
    o = o * sigmoid((h @ get("g1").T) @ get("g2").T).reshape(T, H, e)
    return o.reshape(T, -1) @ get("o").T


def decayed_sums(q, k, v, decay):
    """linear attention: S = decay S + k v^T, o = S^T q, per head"""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    out = np.zeros(v.shape)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out


def lightning(h, get, m, eps):
    T, H = h.shape[0], m["heads"]
    q, k = (silu(h @ get(n).T).reshape(T, H, m["dim"]) for n in "qk")
    v = silu(h @ get("v").T).reshape(T, H, m["vdim"])
    o = rms(decayed_sums(q, k, v, m["decay"]).reshape(T, -1), eps) * get("norm")
    return (o * sigmoid(h @ get("g").T)) @ get("o").T


def layer(x, i, cfg, w, first):
    L, eps, pre = cfg["layers"][i], cfg["norm"]["eps"], "l%d." % i

    def get(name):
        return np.asarray(w[pre + "mix." + name], np.float64)
    h = rms(x, eps) * w[pre + "norm1"]
    m = L["mixer"]
    if L["type"] == "attention":
        x = x + attention(h, get, m, eps, first)
    elif L["type"] == "channel_delta":
        x = x + channel_delta(h, get, m, eps)
    else:
        x = x + lightning(h, get, m, eps)
    if L.get("mlp"):
        h = rms(x, eps) * w[pre + "norm2"]
        x = x + gelu(h @ np.asarray(w[pre + "mlp.up"], np.float64).T) @ np.asarray(w[pre + "mlp.down"], np.float64).T
    return x


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of a whole sequence; streams (a list) receives the
    residual stream after every layer."""
    x = np.asarray(w["embed"], np.float64)[np.asarray(tokens)] * cfg["embedding"]["scale"]
    first = []
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, w, first)
        if streams is not None:
            streams.append(x)
    return (rms(x, cfg["norm"]["eps"]) * w["final.norm"]) @ np.asarray(w["head"], np.float64).T
