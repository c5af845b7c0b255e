"""Fuzuvik without a GPU: the configuration reader, and what the plain
implementation itself makes visible."""
import copy

import numpy as np
import pytest

from tests import fuzuvik_ref as R
from tests.fazinex_util import values
from tests.fuzuvik_util import attention, config, delta, lightning, weights
from vkllama_amd import capi, model as M

BASE = config([delta(4, 2, 16, 24, 3, ff=48), attention(4, 2, 32, rot=16, scaling=(4, 1, 3, 30), size=12, v_mix=True, ff=64),
               lightning([.5, .95, 1.0], 16, 8, ff=40), attention(4, 2, 32, rot=32, base=50.0, size=30, v_mix=True)], 50, 80, scale=2.0)
INVALID = 3


def edit(*path, value):
    cfg = copy.deepcopy(BASE)
    at = cfg
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    return cfg


@pytest.mark.parametrize("path,value", [
    (("vocab",), 0), (("width",), "wide"), (("norm", "eps"), None), (("layers",), []), (("layers", 0, "type"), "conv"),
    (("layers", 0, "mixer", "conv"), 0), (("layers", 0, "mixer", "kv_heads"), 3), (("layers", 0, "mixer", "dim"), None),
    (("layers", 1, "mixer", "scale"), None), (("layers", 1, "mixer", "mask", "size"), 0),
    (("layers", 1, "mixer", "rot", "dims"), 15), (("layers", 1, "mixer", "rot", "dims"), 34),
    (("layers", 1, "mixer", "rot", "scaling", "factor"), 0), (("layers", 1, "mixer", "rot", "scaling", "low"), None),
    (("layers", 1, "mixer", "v_mix"), 1), (("layers", 2, "mixer", "decay"), [.5, .5]),
    (("layers", 2, "mixer", "decay"), [.5, .5, 1.5]), (("layers", 2, "mixer", "decay"), [.5, "x", .5]),
    (("layers", 1, "mlp", "kind"), "sparse"), (("layers", 1, "mlp", "ff"), 0), (("embedding", "scale"), None)])
def test_bad_values_are_named(path, value):
    with pytest.raises(capi.VklError) as e:
        M.CausalModel.create(edit(*path, value=value), weights(BASE))
    assert e.value.code == INVALID and "configuration" in str(e.value)
    keys = [k for k in path if isinstance(k, str)]
    assert keys[-1] in str(e.value) or keys[-2] in str(e.value) or "mixer" in str(e.value)


def test_frequencies():
    plain = R.frequencies({"dims": 8, "base": 100.0})
    assert np.allclose(plain, 100.0 ** (-np.arange(4) / 4))
    sc = R.frequencies({"dims": 8, "base": 100.0, "scaling": {"factor": 10.0, "low": 1.0, "high": 4.0, "original": 40.0}})
    wave = 2 * np.pi / plain                                         # 6.3, 19.9, 62.8, 198.7: kept, blended, slowed, slowed
    assert sc[0] == plain[0] and np.allclose(sc[2:], plain[2:] / 10)
    s = (40 / wave[1] - 1) / 3
    assert np.isclose(sc[1], (1 - s) * plain[1] / 10 + s * plain[1]) and 0 < s < 1


def test_every_mechanism_shows_in_the_logits():
    """The random models of the tests are worth comparing against: leaving out any
    one mechanism of the plain implementation moves the logits by far more than
    the bounds of the comparisons."""
    toks = np.random.default_rng(3).integers(0, 50, 40)
    w = values(weights(BASE, 1))
    want = R.forward(BASE, w, toks)

    def moved(cfg=BASE, ww=w, t=toks, rows=slice(-1, None)):
        d = R.forward(cfg, ww, t)[rows] - want[rows]
        return np.sqrt(np.mean(d * d)) / np.sqrt(np.mean(np.square(want)))

    def without(name, value):
        return moved(ww=dict(w, **{name: value}))

    assert moved() == 0
    assert moved(edit("layers", 1, "mixer", "rot", value=None)) > 0.01
    assert moved(edit("layers", 1, "mixer", "rot", "scaling", value=None)) > 0.005
    assert moved(edit("layers", 3, "mixer", "rot", "base", value=60.0)) > 0.005
    assert moved(edit("layers", 1, "mixer", "mask", "size", value=13)) > 0.01
    assert moved(edit("layers", 3, "mixer", "mask", value=None)) > 0.01
    assert moved(edit("layers", 1, "mixer", "scale", value=0.5)) > 0.01
    assert moved(edit("layers", 3, "mixer", "v_mix", value=False)) > 0.01
    assert moved(edit("layers", 2, "mixer", "decay", value=[.6, .95, 1.0])) > 0.005
    assert moved(edit("layers", 2, "mlp", value=None)) > 0.05
    assert moved(edit("embedding", "scale", value=1.0)) > 0.02
    assert moved(edit("norm", "eps", value=0.3)) > 0.02
    for n in ("l0.mix.a2", "l0.mix.dt_bias", "l0.mix.b", "l0.mix.g2", "l2.mix.g", "l3.mix.vmix", "l0.mix.A_log"):
        assert without(n, np.zeros_like(w[n])) > 0.003, n
    for n in ("l0.mix.norm", "l2.mix.norm", "l1.norm2", "l2.norm1", "final.norm"):
        assert without(n, np.ones_like(w[n])) > 0.02, n
    first = w["l0.mix.k.conv"].copy()
    first[:, 0] = 0
    assert without("l0.mix.k.conv", first) > 0.01
    assert without("l1.mix.vmix", np.float64(0.9)) == 0                # (the first mixing layer mixes nothing)
    t2 = toks.copy()
    t2[0] = (t2[0] + 1) % 50                                           # a token far back: through the states alone
    assert moved(t=t2) > 0.001


def test_the_sink_takes_part_of_the_weight():
    assert np.isclose(R.sink_softmax(np.array([0.0])).sum(), 0.5)
    assert np.isclose(R.sink_softmax(np.array([50.0, 50.0])).sum(), 1.0)
    assert R.sink_softmax(np.array([-50.0])).sum() < 1e-20
    assert np.isfinite(R.sink_softmax(np.array([900.0, -900.0]))).all()
