"""Plain float64 implementation of the Fazinex decoder, one function per
mechanism, written from the equations.  It shares no code with the product and
is slow on purpose: attention walks queries one by one over full score rows,
and nothing is cached.

A model is (cfg, w): cfg the decoded config.json, w a dict name -> array."""
import math

import numpy as np


def rms_norm(x, w, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * np.asarray(w, np.float64)


def softmax(s):
    e = np.exp(s - np.max(s))
    return e / e.sum()


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def query_temperature(p, coef, every):
    return 1.0 + coef * math.log(math.floor((p + 1) / every) + 1.0)


def causal_attention(q, k, v, scale):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; runs of H / G query
    heads share a key/value head, a row attends to itself and what came before."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            out[i, h] = softmax(k[: i + 1, g] @ q[i, h] * scale) @ v[: i + 1, g]
    return out


def shared_kv_attention(h, get, m):
    """One projection serves as keys and as values; besides the mask, positions
    enter through a factor on the queries."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q = (h @ get("q").T).reshape(T, H, d)
    k = (h @ get("k").T).reshape(T, G, d)
    t = m.get("q_temp")
    if t:
        q = q * np.array([query_temperature(p, t["coef"], t["every"]) for p in range(T)])[:, None, None]
    return causal_attention(q, k, k, m["scale"]).reshape(T, -1) @ get("o").T


def latent_attention(h, get, m, eps):
    """Keys and values are expanded from a normed latent row; each head's
    output is scaled by its own sigmoid gate."""
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    q = (h @ get("q").T).reshape(T, H, d)
    c = rms_norm(h @ get("dkv").T, get("dkv.norm"), eps)
    k = (c @ get("uk").T).reshape(T, H, d)
    v = (c @ get("uv").T).reshape(T, H, e)
    o = causal_attention(q, k, v, m["scale"])
    o = o * sigmoid(h @ get("g").T)[:, :, None]
    return o.reshape(T, -1) @ get("o").T


def dense_ff(h, up, down):
    return np.square(np.maximum(h @ up.T, 0.0)) @ down.T


def layer_order(cfg):
    """Layer numbers in the order they run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def layer(x, i, cfg, w):
    L, eps, pre = cfg["layers"][i], cfg["norm"]["eps"], "l%d." % i
    h = rms_norm(x, w[pre + "norm1"], eps)

    def get(name):
        return np.asarray(w[pre + "mix." + name], np.float64)
    m = L["mixer"]
    y = latent_attention(h, get, m, eps) if L["type"] == "latent_attention" else shared_kv_attention(h, get, m)
    if L.get("mlp"):
        y = y + dense_ff(h, np.asarray(w[pre + "mlp.up"], np.float64), np.asarray(w[pre + "mlp.down"], np.float64))
    return x + y


def softcap(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of a whole sequence; streams (a list) receives the
    residual stream after every layer that ran."""
    eps = cfg["norm"]["eps"]
    emb = np.asarray(w["embed"], np.float64)
    x = rms_norm(emb[np.asarray(tokens)], w["embed.norm"], eps)
    for i in layer_order(cfg):
        x = layer(x, i, cfg, w)
        if streams is not None:
            streams.append(x)
    return softcap(rms_norm(x, w["final.norm"], eps) @ emb.T, cfg.get("logit_softcap"))
