"""Fazinex without a GPU: the configuration reader, the C ABI's coverage, and
what the plain implementation itself makes visible."""
import copy
import ctypes as C
import json

import numpy as np
import pytest

from tests import fazinex_ref as R
from tests.fazinex_util import attention, config, latent, save, values, weights
from tests.test_capi_cpu import _declared
from vkllama_amd import capi, model as M, stack as K

BASE = config([attention(4, 2, 32, q_temp=(0.4, 8), ff=64), latent(3, 16, 24, 40, ff=48)], 50, 80, loop=(0, 2, 2))
INVALID, NOT_FOUND, UNIMPLEMENTED = 3, 5, 12


def create(cfg):
    try:
        M.CausalModel.create(cfg, weights(BASE)).close()
    except capi.VklError as e:
        return e.code, str(e)
    return 0, ""


def test_stack_header_is_bound():
    names = _declared("vkl_stack.h")
    assert sorted(K.SIGNATURES) == names
    lib = K.lib()
    for n in names:
        assert hasattr(lib, n), n


@pytest.mark.parametrize("text,code", [("{", INVALID), ("[]", INVALID), ('{"architecture": 3}', INVALID),
                                       ('{"architecture": "Nothing"}', UNIMPLEMENTED), ('{"a": "\\ud800"}', INVALID),
                                       ('{"architecture": "Fazinex"} x', INVALID)])
def test_unreadable_configurations(text, code):
    assert create(text)[0] == code


@pytest.mark.parametrize("path,value", [
    (("vocab",), 0), (("width",), "wide"), (("norm", "eps"), None), (("layers",), []), (("layers", 0, "type"), "conv"),
    (("layers", 0, "mixer", "heads"), 2.5), (("layers", 0, "mixer", "kv_heads"), 3), (("layers", 0, "mixer", "scale"), None),
    (("layers", 0, "mixer", "q_temp", "every"), 0), (("layers", 0, "mlp", "kind"), "sparse"),
    (("layers", 1, "mixer", "kv_rank"), 0), (("loop", "stop"), 3), (("loop", "times"), 0), (("loop", "start"), -1),
    (("logit_softcap",), -1.0)])
def test_bad_values_are_named(path, value):
    cfg = copy.deepcopy(BASE)
    at = cfg
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    code, msg = create(cfg)
    assert code in (INVALID, UNIMPLEMENTED) and "configuration" in msg
    assert [k for k in path if isinstance(k, str)][-1] in msg or "mixer" in msg or "kind" in msg or "loop" in msg


def test_paths_that_hold_no_model(tmp_path):
    def load(path, **kw):
        with pytest.raises(capi.VklError) as e:
            M.CausalModel.load(path, **kw)
        return e.value.code
    assert load(tmp_path / "nowhere") == NOT_FOUND
    assert load(tmp_path) == NOT_FOUND
    (tmp_path / "config.json").write_text(json.dumps(BASE))
    assert load(tmp_path) == NOT_FOUND
    (tmp_path / "model.safetensors").write_bytes(b"\xff" * 64)
    assert load(tmp_path) == INVALID
    save(str(tmp_path), BASE, weights(BASE))
    data = (tmp_path / "model.safetensors").read_bytes()
    (tmp_path / "model.safetensors").write_bytes(data[:-1])               # offsets beyond the end
    assert load(tmp_path) == INVALID
    out = C.c_void_p()
    assert M.lib().vkl_model_load(0, str(tmp_path).encode(), b"int4", 0, C.byref(out)) == INVALID
    assert M.lib().vkl_model_forward_rows(None, None, 0, 0, None, 0, None) == INVALID
    assert M.lib().vkl_model_context_length(None) == 0


def test_layers_run_in_the_order_of_the_loop():
    assert R.layer_order(dict(BASE, layers=[{}] * 5, loop={"start": 1, "stop": 3, "times": 3})) \
        == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert R.layer_order(dict(BASE, layers=[{}] * 3, loop=None)) == [0, 1, 2]


def test_every_mechanism_shows_in_the_logits():
    """The random models of the tests are worth comparing against: leaving out any
    one mechanism of the plain implementation moves the logits by far more than
    the bounds of the comparisons."""
    toks = np.random.default_rng(3).integers(0, 50, 40)
    w = values(weights(BASE, 1))
    want = R.forward(BASE, w, toks)

    def moved(cfg=BASE, ww=w, t=toks):
        return np.sqrt(np.mean(np.square(R.forward(cfg, ww, t)[-1] - want[-1]))) / np.sqrt(np.mean(np.square(want)))

    def edit(*path, value):
        cfg = copy.deepcopy(BASE)
        at = cfg
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        return cfg

    assert moved() == 0
    assert moved(edit("layers", 0, "mixer", "q_temp", value=None)) > 0.05
    assert moved(edit("layers", 0, "mixer", "q_temp", "every", value=9)) > 0.005
    assert moved(edit("loop", value=None)) > 0.1
    assert moved(edit("layers", 1, "mlp", value=None)) > 0.1
    assert moved(edit("norm", "eps", value=0.3)) > 0.05
    assert moved(edit("logit_softcap", value=2.0)) > 0.05
    for name in ("l1.mix.g", "l1.mix.dkv.norm", "embed.norm", "l0.norm1", "l0.mix.k", "l1.mix.uk"):
        ww = dict(w)
        ww[name] = np.ones_like(w[name]) if w[name].ndim == 1 else np.zeros_like(w[name])
        assert moved(ww=ww) > 0.02, name
    t2 = toks.copy()
    t2[0] = (t2[0] + 1) % 50                                             # a token far back
    assert moved(t=t2) > 0.02
