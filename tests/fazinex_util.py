"""Small Fazinex configurations and random weights for the tests."""
import json
import os

import numpy as np


def bf16_bits(a):
    """float array -> bf16 bits, rounded to nearest even"""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_values(bits):
    return (np.asarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def attention(heads, kv_heads, dim, scale=None, q_temp=None, ff=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or dim ** -0.5}
    if q_temp:
        m["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def latent(heads, dim, vdim, rank, scale=None, ff=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale or dim ** -0.5},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab, width, loop=None, cap=30.0, eps=1e-5):
    return {"architecture": "Fazinex", "layers": layers, "vocab": vocab, "width": width, "norm": {"eps": eps},
            "loop": loop and {"start": loop[0], "stop": loop[1], "times": loop[2]}, "logit_softcap": cap}


def tensor_shapes(cfg):
    w, shapes = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "embed.norm": (cfg["width"],),
                               "final.norm": (cfg["width"],)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], "l%d." % i
        shapes[p + "norm1"] = (w,)
        shapes[p + "mix.q"] = (m["heads"] * m["dim"], w)
        shapes[p + "mix.o"] = (w, m["heads"] * m["vdim"])
        if L["type"] == "attention":
            shapes[p + "mix.k"] = (m["kv_heads"] * m["dim"], w)
        else:
            shapes[p + "mix.dkv"] = (m["kv_rank"], w)
            shapes[p + "mix.dkv.norm"] = (m["kv_rank"],)
            shapes[p + "mix.uk"] = (m["heads"] * m["dim"], m["kv_rank"])
            shapes[p + "mix.uv"] = (m["heads"] * m["vdim"], m["kv_rank"])
            shapes[p + "mix.g"] = (m["heads"], w)
        if L.get("mlp"):
            shapes[p + "mlp.up"] = (L["mlp"]["ff"], w)
            shapes[p + "mlp.down"] = (w, L["mlp"]["ff"])
    return shapes


def weights(cfg, seed=0):
    """name -> bf16 bits: matrices N(0, 1/sqrt(inputs)), norms around 1"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, sh in tensor_shapes(cfg).items():
        if len(sh) == 1:
            a = rng.uniform(0.6, 1.4, sh)
        else:
            a = rng.standard_normal(sh) / np.sqrt(sh[1])
        out[name] = bf16_bits(a)
    return out


def values(w):
    return {k: bf16_values(v).astype(np.float64) for k, v in w.items()}


def save(folder, cfg, w):
    """config.json and model.safetensors"""
    head, data = {}, b""
    for name, a in w.items():
        head[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [len(data), len(data) + a.nbytes]}
        data += a.tobytes()
    text = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(len(text).to_bytes(8, "little") + text + data)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)


def row_errors(got, want):
    """per row: rms of the difference (mean taken off) over the rms of all wanted logits"""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / np.sqrt(np.mean(np.square(want)))


# rounding alone: 32-bit, and bf16 products and activations
LIMIT = {"float32": 3e-5, "bfloat16": 3e-2}
