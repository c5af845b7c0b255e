"""Small Fuzuvik configurations and random weights for the tests."""
import numpy as np

from tests.fazinex_util import bf16_bits


def attention(heads, kv_heads, dim, vdim=None, rot=None, base=1e4, scaling=None, size=None, scale=None, v_mix=False, ff=None):
    """rot: rotated values per head; scaling: (factor, low, high, original)"""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim or dim, "scale": scale or dim ** -0.5, "v_mix": v_mix,
         "mask": {"size": size} if size else None}
    if rot:
        m["rot"] = {"base": base, "dims": rot,
                    "scaling": scaling and dict(zip(("factor", "low", "high", "original"), scaling))}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads, kv_heads, dim, vdim, conv=4, ff=None, ranks=(8, 8)):
    return {"type": "channel_delta", "ranks": ranks,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def lightning(decay, dim, vdim, ff=None):
    return {"type": "lightning", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab, width, scale=1.0, eps=1e-5):
    return {"architecture": "Fuzuvik", "layers": layers, "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}}


def tensor_shapes(cfg):
    w = cfg["width"]
    shapes = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], "l%d." % i
        H, d, e = m["heads"], m["dim"], m["vdim"]
        G = m.get("kv_heads", H)
        shapes[p + "norm1"] = (w,)
        shapes[p + "mix.q"], shapes[p + "mix.k"] = ((H if L["type"] == "attention" else G) * d, w), (G * d, w)
        shapes[p + "mix.v"] = ((G if L["type"] == "attention" else H) * e, w)
        shapes[p + "mix.o"] = (w, H * e)
        if L["type"] == "attention":
            if m["v_mix"]:
                shapes[p + "mix.vmix"] = ()
        elif L["type"] == "channel_delta":
            ra, rg = L["ranks"]
            for n, c in (("q", G * d), ("k", G * d), ("v", H * e)):
                shapes[p + "mix.%s.conv" % n] = (c, m["conv"])
            shapes.update({p + "mix.b": (H, w), p + "mix.A_log": (H,), p + "mix.norm": (e,), p + "mix.a1": (ra, w),
                           p + "mix.a2": (H * d, ra), p + "mix.dt_bias": (H * d,), p + "mix.g1": (rg, w),
                           p + "mix.g2": (H * e, rg)})
        else:
            shapes.update({p + "mix.g": (H * e, w), p + "mix.norm": (H * e,)})
        if L["mlp"]:
            shapes[p + "norm2"] = (w,)
            shapes[p + "mlp.up"] = (L["mlp"]["ff"], w)
            shapes[p + "mlp.down"] = (w, L["mlp"]["ff"])
    return shapes


def weights(cfg, seed=0):
    """name -> bf16 bits: matrices N(0, 1/sqrt(inputs)), norms around 1, decays from
    almost none to strong"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, sh in tensor_shapes(cfg).items():
        if name.endswith("A_log"):
            a = rng.uniform(-4.0, 1.5, sh)
        elif name.endswith("dt_bias"):
            a = rng.uniform(-5.0, 2.0, sh)
        elif name.endswith("vmix"):
            a = np.array(0.375)
        elif len(sh) == 1:
            a = rng.uniform(0.6, 1.4, sh)
        else:
            a = rng.standard_normal(sh) / np.sqrt(sh[1])
        out[name] = bf16_bits(a).reshape(sh)
    return out
