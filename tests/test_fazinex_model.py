"""The Fazinex decoder on the GPU, through the C ABI, against the plain
implementation in tests/fazinex_ref.py: whole prompts, portions, single tokens,
both number formats, generation, and the programs around it."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests import fazinex_ref as R
from tests.fazinex_util import LIMIT, attention, config, latent, row_errors, save, values, weights
from vkllama_amd import capi, model as M

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# sizes on and off every padding; one and several key/value heads; loops over one
# layer, over all, and none; layers without a feed-forward part; with and without
# the soft cap and the query factor
CONFIGS = {
    "mixed": config([attention(6, 2, 48, q_temp=(0.4, 16), ff=100), latent(5, 24, 40, 72, ff=72), attention(4, 4, 32, ff=33),
                     latent(3, 64, 32, 64)], 131, 144, loop=(1, 3, 3)),
    "one-layer-loop": config([latent(2, 96, 96, 200, ff=256), attention(8, 1, 80, ff=512)], 256, 128, loop=(1, 2, 2), cap=None),
    "all-looped": config([attention(3, 3, 16, q_temp=(0.9, 5), ff=40)], 67, 40, loop=(0, 1, 4), cap=5.0, eps=1e-2),
    "wide": config([attention(9, 3, 160, ff=1000), latent(16, 128, 64, 512, ff=700)], 517, 2112, loop=None),
    "big-heads": config([attention(4, 2, 288, ff=64), latent(3, 300, 20, 600, ff=96), attention(2, 2, 520)], 97, 160,
                        loop=(1, 3, 2)),
    "no-mlp": config([latent(1, 8, 8, 8), attention(1, 1, 8)], 33, 24, loop=(0, 2, 1)),
}
# scores far apart: every query depends on few keys, anywhere in its past
PEAKED = config([attention(4, 2, 32, scale=1.2, q_temp=(0.3, 100), ff=64), latent(4, 32, 32, 64, scale=1.2, ff=64)], 200, 128,
                loop=(0, 1, 2))
DTYPES = ["float32", "bfloat16"]
_cache = {}


def case(name, n=90):
    """(cfg, weights, tokens, logits of the plain implementation)"""
    if (name, n) not in _cache:
        cfg = PEAKED if name == "peaked" else CONFIGS[name]
        w = weights(cfg, seed=len(name))
        toks = np.random.default_rng(n).integers(0, cfg["vocab"], n).astype(np.uint32)
        streams = []
        _cache[name, n] = cfg, w, toks, R.forward(cfg, values(w), toks, streams), streams
    return _cache[name, n]


def run(m, toks, cuts, start=0):
    """logits of every position, the sequence cut at `cuts`"""
    out, at = [], start
    for n in cuts:
        out.append(m.forward_rows(toks[at - start:at - start + n], at, np.arange(n)))
        at += n
    return np.concatenate(out)


def check(got, want, dtype, factor=1.0):
    e = row_errors(got, want)
    assert e.max() < LIMIT[dtype] * factor, (int(e.argmax()), float(e.max()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_residual_stream_and_whole_prompt(name, dtype):
    cfg, w, toks, want, streams = case(name)
    m = M.CausalModel.create(cfg, w, dtype, 128)
    got = m.residual_streams(toks, 0, len(streams), cfg["width"])
    for i, (g, s) in enumerate(zip(got, streams)):
        assert np.abs(g - s).max() < LIMIT[dtype] * np.abs(s).max(), i
    check(run(m, toks, [len(toks)]), want, dtype)
    # rows in any order, and none at all
    rows = np.array([5, 80, 5, 0], np.uint32)
    check(m.forward_rows(toks, 0, rows), want[rows], dtype)
    assert m.forward_rows(toks, 0, np.empty(0, np.uint32)).shape == (0, cfg["vocab"])
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("fused", [1, 0])
def test_token_by_token(name, dtype, fused):
    """From an empty cache to its last row, on the fused step and on the operators."""
    cfg, w, toks, want, _ = case(name)
    m = M.CausalModel.create(cfg, w, dtype, len(toks))
    m.set_option("fused_decode", fused)
    check(run(m, toks, [1] * len(toks)), want, dtype)
    with pytest.raises(capi.VklError):
        m.forward([1], len(toks))
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[2] * 45, [3, 2, 17, 16, 33, 2, 17], [64, 2, 24], [1, 63, 1, 25], [16, 17, 57]])
def test_portions(cuts, dtype):
    cfg, w, toks, want, _ = case("mixed")
    m = M.CausalModel.create(cfg, w, dtype, 90)
    check(run(m, toks, cuts), want, dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys_in_prompts_portions_and_decoding(dtype):
    """A sequence past several tiles and splits, whose queries each pick out few
    keys of their whole past: prompt, prompt in portions, and single tokens over
    the long context, each from the cache rows another sequence left."""
    cfg, w, toks, want, _ = case("peaked", 700)
    m = M.CausalModel.create(cfg, w, dtype, 701)
    f = 4.0 if dtype == "bfloat16" else 3.0                         # (peaked scores amplify rounding)
    check(run(m, toks, [700]), want, dtype, f)
    other = (toks[::-1] + 7) % cfg["vocab"]
    m.forward_rows(other, 0, [0])
    check(run(m, toks, [130, 2, 200, 5, 16, 17, 330]), want, dtype, f)
    m.forward_rows(other, 0, [0])
    got = np.concatenate([run(m, toks[:560], [560]), run(m, toks[560:], [1] * 140, 560)])
    check(got, want, dtype, f)
    # a shorter request on the rows of the longer one
    check(run(m, toks[:40], [20] + [1] * 20), want[:40], dtype, f)
    m.close()


def test_formats_keep_the_step_and_the_prompt_pass_together():
    """Both paths of one model, position by position: closer to one another than
    either bound, so that a cut of the prompt does not show."""
    cfg, w, toks, _, _ = case("mixed")
    m = M.CausalModel.create(cfg, w, "float32", 90)
    a, b, c = run(m, toks, [90]), run(m, toks, [1] * 90), run(m, toks, [45, 45])
    assert row_errors(b, a).max() < 1e-5 and row_errors(c, a).max() < 1e-5
    m.close()


def greedy_plain(cfg, w, prompt, n):
    toks, margins, v = list(prompt), [], values(w)
    for _ in range(n):
        z = R.forward(cfg, v, np.array(toks))[-1]
        s = np.sort(z)
        margins.append((s[-1] - s[-2]) / np.sqrt(np.mean(z * z)))
        toks.append(int(np.argmax(z)))
    return toks[len(prompt):], margins


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_prompt", [1, 9])
def test_greedy_generation(dtype, n_prompt):
    """The token loop, replayed from a graph and step by step, on the fused step
    and on the operators, against the plain implementation's choices; several
    generations in a row, with other work between them."""
    cfg, w, toks, _, _ = case("mixed")
    prompt, n = toks[:n_prompt], 24
    want, margins = greedy_plain(cfg, w, prompt, n)
    sure = next((i for i, g in enumerate(margins) if g < 4 * LIMIT[dtype]), n)   # (a near-tie ends the comparison)
    m = M.CausalModel.create(cfg, w, dtype, 64)
    first = None
    for graph, fused in ((1, 1), (1, 1), (0, 1), (1, 1), (0, 0)):
        m.set_option("decode_graph", graph)
        m.set_option("fused_decode", fused)
        ids, _, _ = m.generate_greedy(prompt, n)
        assert list(ids[:sure]) == want[:sure], (graph, fused)
        if fused:
            assert first is None or list(ids) == first               # the same launches: the same bits
            first = list(ids)
        m.forward(toks[:30], 0)
    with pytest.raises(capi.VklError):
        m.generate_greedy(prompt, 65)
    m.close()
    assert sure >= 8 or dtype == "bfloat16"


def test_sampled_generation_replays_and_follows_its_seed():
    cfg, w, toks, _, _ = case("mixed")
    m = M.CausalModel.create(cfg, w, "bfloat16", 80)
    a, _, _ = m.generate_sampled(toks[:6], 40, topk=20, seed=5)
    m.set_option("decode_graph", 0)
    b, _, _ = m.generate_sampled(toks[:6], 40, topk=20, seed=5)
    m.set_option("decode_graph", 1)
    c, _, _ = m.generate_sampled(toks[:6], 40, topk=20, seed=6)
    d, _, _ = m.generate_sampled(toks[:6], 40, topp=0.9, seed=5)
    g, _, _ = m.generate_greedy(toks[:6], 40)
    h, _, _ = m.generate_sampled(toks[:6], 40, topk=1, seed=9)
    assert list(a) == list(b) and list(a) != list(c) and list(g) == list(h) and len(set(d)) > 5
    # every drawn token was among the candidates of its step
    seq = list(toks[:6]) + [int(t) for t in a]
    m.set_option("fused_decode", 1)
    z = m.forward_rows(seq[:-1], 0, np.arange(5, 45))
    for row, t in zip(z, a):
        assert np.sum(row > row[t]) < 24                              # (20, with room for rounding)
    m.close()


def test_two_models_at_once_keep_their_own_state():
    cfg, w, toks, want, _ = case("mixed")
    cfg2, w2, toks2, want2, _ = case("one-layer-loop")
    a, b = M.CausalModel.create(cfg, w, "float32", 90), M.CausalModel.create(cfg2, w2, "float32", 90)
    ids = a.generate_greedy(toks[:4], 20)[0], b.generate_greedy(toks2[:4], 20)[0]
    for i in range(90):
        check(a.forward_rows([toks[i]], i, [0]), want[i:i + 1], "float32", 3)
        check(b.forward_rows([toks2[i]], i, [0]), want2[i:i + 1], "float32", 3)
    assert list(a.generate_greedy(toks[:4], 20)[0]) == list(ids[0])
    a.close()
    assert list(b.generate_greedy(toks2[:4], 20)[0]) == list(ids[1])
    b.close()


def test_decode_step_bytes_counts_weights_and_cache():
    cfg, w, _, _, _ = case("one-layer-loop")
    m = M.CausalModel.create(cfg, w, "bfloat16", 32)
    per_pos = m.decode_step_bytes(11) - m.decode_step_bytes(10)
    assert per_pos == 2 * (256 + 2 * 96)                              # a padded latent row and, twice, a padded key row
    assert m.decode_step_bytes(10) > sum(a.nbytes for a in w.values())
    assert m.context_length() == 32
    m.close()


def test_unaligned_tensors_missing_tensors_and_other_families(tmp_path):
    cfg, w, toks, want, _ = case("no-mlp", 30)
    save(str(tmp_path), cfg, w)
    m = M.CausalModel.load(tmp_path, "float32", 40)
    check(run(m, toks, [30]), want, "float32")
    buf = np.empty(8, np.uint16)
    assert M.lib().vkl_model_read_kv_cache(m._h, 0, 0, buf.ctypes.data, 8) == 12
    with pytest.raises(capi.VklError):
        m.set_option("decode_mode", 1)                                # an option of another family
    m.close()
    short = {k: v for k, v in w.items() if k != "l1.mix.k"}
    with pytest.raises(capi.VklError) as e:
        M.CausalModel.create(cfg, short, None, 40)
    assert "l1.mix.k" in str(e.value)
    bad = dict(w, **{"l0.mix.uv": w["l0.mix.uv"][:, :-1]})
    with pytest.raises(capi.VklError) as e:
        M.CausalModel.create(cfg, bad, None, 40)
    assert "l0.mix.uv" in str(e.value)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_program(tmp_path, dtype):
    """bin/trace_run: requests one after the other, in portions, with and without
    wanted logits."""
    cfg, w, toks, want, _ = case("mixed")
    save(str(tmp_path), cfg, w)
    out = tmp_path / "logits"
    steps = [{"step": 0, "entries": [{"id": "u", "tokens": toks[:50].tolist(), "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "u", "tokens": toks[50:53].tolist(), "want": [2, 0]}], "end": []},
             {"step": 2, "entries": [{"id": "u", "tokens": toks[53:54].tolist(), "want": [0]}], "end": ["u"]},
             {"step": 9, "entries": [{"id": "v", "tokens": toks[:7].tolist(), "want": [6]}], "end": ["v"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out",
                        str(out), "--max-tokens", "60"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-800:]
    assert r.stdout.split("\n")[:4] == ["done 0", "done 1", "done 2", "done 9"]
    assert sorted(os.listdir(out)) == ["1.f32", "2.f32", "9.f32"]
    for step, rows in ((1, [52, 50]), (2, [53]), (9, [6])):
        check(np.fromfile(out / ("%d.f32" % step), "<f4").reshape(len(rows), -1), want[rows], dtype, 2)
    mixed = [dict(steps[0]), dict(steps[3])]                           # the first request is still live
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out",
                        str(out), "--max-tokens", "60"], input="\n".join(json.dumps(s) for s in mixed) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert r.returncode != 0 and "one sequence" in r.stderr


def test_command_lines_generate(tmp_path):
    cfg, w, toks, _, _ = case("mixed")
    save(str(tmp_path), cfg, w)
    m = M.CausalModel.create(cfg, w, "float32", 64)
    want = [int(t) for t in m.generate_greedy(toks[:5], 10)[0]]
    m.close()
    ids = [str(t) for t in toks[:5]]
    r = subprocess.run([sys.executable, "-m", "vkllama_amd.infer", str(tmp_path), "10", "--dtype", "float32",
                        "--max-tokens", "64", "--ids"] + ids, capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-800:]
    assert [int(t) for t in r.stdout.split("ids:")[1].split()] == want
    r = subprocess.run([os.path.join(ROOT, "vkllama_amd", "lib", "llama2_infer"), "--dtype", "float32", "--max-tokens",
                        "64", str(tmp_path), "10"] + ids, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-800:]
    assert [int(t) for t in r.stdout.split()] == want
