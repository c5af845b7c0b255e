"""The Fuzuvik decoder on the GPU, through the C ABI, against the plain
implementation in tests/fuzuvik_ref.py: whole prompts, portions, single tokens,
both number formats, generation, and the programs around it."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests import fuzuvik_ref as R
from tests.fazinex_util import LIMIT, row_errors, save, values
from tests.fuzuvik_util import attention, config, delta, lightning, weights
from vkllama_amd import capi, model as M

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# sizes on and off every padding, every mixer first, last, alone and twice, shared
# and unshared heads, with and without rotation, scaling, chunks, mixed values and
# feed-forward parts
CONFIGS = {
    "mixed": config([delta(4, 2, 48, 40, 3, ff=100, ranks=(24, 40)), lightning([.5, .9, .99], 24, 40, ff=72),
                     attention(4, 2, 40, 24, rot=24, size=37, v_mix=True, ff=64),
                     attention(2, 2, 40, 24, rot=40, scaling=(6, 0.8, 5, 70), size=11, v_mix=True),
                     lightning([1.0, .1], 96, 72)], 131, 144, scale=3.0),
    "attention-only": config([attention(6, 3, 32, size=16, scale=0.9, ff=33), attention(6, 3, 32, rot=8, base=50, size=64, v_mix=True),
                              attention(3, 3, 80, 32, size=1, v_mix=True, ff=40), attention(9, 3, 20, 32, rot=20, v_mix=True)], 67, 40, eps=1e-2),
    "delta-first-last": config([delta(3, 3, 32, 32, 4, ff=64, ranks=(64, 128)), attention(2, 1, 64, size=50, ff=96),
                                delta(6, 2, 72, 100, 1, ranks=(5, 130)), delta(2, 1, 128, 64, 6, ff=48)], 256, 128, scale=0.5),
    "sums-only": config([lightning([.3, .6, .8, .95, 1.0], 20, 52), lightning([.999], 100, 33, ff=17)], 33, 72),
    "wide": config([lightning(np.linspace(.5, .999, 12), 128, 128, ff=1000), delta(8, 4, 96, 160, 4, ff=700, ranks=(128, 64)),
                    attention(10, 2, 160, 128, rot=96, base=1e5, scaling=(4, 1, 2, 900), size=60, v_mix=True, ff=900)], 517, 2112),
    "big-heads": config([delta(2, 1, 200, 224, 2, ff=64), attention(4, 2, 288, rot=100, size=30, ff=64),
                         lightning([.9, .99], 256, 136), attention(2, 1, 520, 260, size=80, v_mix=True)], 97, 160),
}
# scores far apart: every query of the attention depends on few keys of its chunk, and
# the recurrences hardly forget
PEAKED = config([delta(4, 2, 32, 32, 3, ff=64), attention(4, 2, 64, rot=32, base=300.0, size=90, scale=0.6, v_mix=True, ff=64),
                 lightning([1.0, .999, .9], 32, 32, ff=64), attention(4, 2, 32, 64, size=250, scale=0.9, v_mix=True)], 200, 128)
DTYPES = ["float32", "bfloat16"]
_cache = {}


def case(name, n=90):
    """(cfg, weights, tokens, logits of the plain implementation, residual streams)"""
    if (name, n) not in _cache:
        cfg = PEAKED if name == "peaked" else CONFIGS[name]
        w = weights(cfg, seed=len(name))
        if name == "peaked":
            w["l0.mix.A_log"] = np.full_like(w["l0.mix.A_log"], 0xC0C0)   # e^-6: a long memory
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
    rows = np.array([5, 80, 5, 0], np.uint32)
    check(m.forward_rows(toks, 0, rows), want[rows], dtype)
    assert m.forward_rows(toks, 0, np.empty(0, np.uint32)).shape == (0, cfg["vocab"])
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("fused", [1, 0])
def test_token_by_token(name, dtype, fused):
    """From the first position to the last row of the caches, on the fused step and
    on the operators."""
    cfg, w, toks, want, _ = case(name)
    m = M.CausalModel.create(cfg, w, dtype, len(toks))
    m.set_option("fused_decode", fused)
    check(run(m, toks, [1] * len(toks)), want, dtype)
    with pytest.raises(capi.VklError):
        m.forward([1], len(toks))
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "delta-first-last"])
@pytest.mark.parametrize("cuts", [[2] * 45, [3, 2, 17, 16, 33, 2, 17], [64, 2, 24], [1, 63, 1, 25], [36, 2, 35, 1, 2, 14],
                                  [65, 25], [24, 23, 43]])
def test_portions(name, cuts, dtype):
    cfg, w, toks, want, _ = case(name)
    m = M.CausalModel.create(cfg, w, dtype, 90)
    check(run(m, toks, cuts), want, dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys_chunk_edges_and_long_decoding(dtype):
    """A sequence past several tiles, chunks and splits, whose queries pick out few
    keys: prompt, prompt in portions that end just before, at and just after a
    chunk's edge, and long decoding over such edges, each on what another sequence
    left behind."""
    cfg, w, toks, want, _ = case("peaked", 620)
    m = M.CausalModel.create(cfg, w, dtype, 621)
    f = 6.0                                                         # (peaked scores amplify rounding)
    check(run(m, toks, [620]), want, dtype, f)
    other = (toks[::-1] + 7) % cfg["vocab"]
    m.forward_rows(other, 0, [0])
    check(run(m, toks, [89, 2, 88, 1, 70, 2, 17, 231, 2, 118]), want, dtype, f)
    m.forward_rows(other, 0, [0])
    got = np.concatenate([run(m, toks[:170], [170]), run(m, toks[170:], [1] * 450, 170)])
    check(got, want, dtype, f)
    # a shorter request after the longer one: nothing of it may be left
    check(run(m, toks[:40], [20] + [1] * 20), want[:40], dtype, f)
    m.close()


def test_a_cut_of_the_prompt_does_not_show():
    """All ways through one model, position by position: closer to one another than
    to the plain implementation's bound."""
    cfg, w, toks, _, _ = case("mixed")
    m = M.CausalModel.create(cfg, w, "float32", 90)
    a = run(m, toks, [90])
    for cuts in ([1] * 90, [45, 45], [23, 24, 2, 41]):
        assert row_errors(run(m, toks, cuts), a).max() < 1e-5
    m.close()


def test_a_state_has_one_position():
    """Rows of a cache can be read anywhere, a recurrent state only where it is: a
    pass that neither continues the last one nor starts a sequence is refused."""
    cfg, w, toks, want, _ = case("mixed")
    m = M.CausalModel.create(cfg, w, "float32", 90)
    run(m, toks, [40])
    for offset in (39, 41, 20):
        with pytest.raises(capi.VklError):
            m.forward([3], offset)
        run(m, toks, [40])
    check(run(m, toks[40:], [20, 1, 1], 40), want[40:62], "float32")
    ids, _, _ = m.generate_greedy(toks[:5], 8)
    seq = list(toks[:5]) + [int(t) for t in ids]
    a = m.forward_rows([seq[12]], 12, [0])                          # the last id, behind the generation
    check(a, m.forward_rows(seq, 0, [12]), "float32")
    m.close()
    # without a state the positions are free
    cfg, w, toks, want, _ = case("attention-only")
    m = M.CausalModel.create(cfg, w, "float32", 90)
    run(m, toks, [90])
    check(m.forward_rows(toks[30:32], 30, [0, 1]), want[30:32], "float32")
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
    prompt, n = toks[:n_prompt], 40
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
    g, _, _ = m.generate_greedy(toks[:6], 40)
    h, _, _ = m.generate_sampled(toks[:6], 40, topk=1, seed=9)
    assert list(a) == list(b) and list(a) != list(c) and list(g) == list(h)
    m.close()


def test_two_models_at_once_keep_their_own_state():
    cfg, w, toks, want, _ = case("mixed")
    cfg2, w2, toks2, want2, _ = case("sums-only")
    a, b = M.CausalModel.create(cfg, w, "float32", 90), M.CausalModel.create(cfg2, w2, "float32", 90)
    ids = a.generate_greedy(toks[:4], 20)[0], b.generate_greedy(toks2[:4], 20)[0]
    for i in range(60):
        check(a.forward_rows([toks[i]], i, [0]), want[i:i + 1], "float32", 3)
        check(b.forward_rows([toks2[i]], i, [0]), want2[i:i + 1], "float32", 3)
    assert list(a.generate_greedy(toks[:4], 20)[0]) == list(ids[0])
    a.close()
    assert list(b.generate_greedy(toks2[:4], 20)[0]) == list(ids[1])
    b.close()


def test_decode_step_bytes_count_weights_rows_of_the_chunk_and_states():
    cfg, w, _, _, _ = case("mixed")
    m = M.CausalModel.create(cfg, w, "bfloat16", 90)
    per_pos = m.decode_step_bytes(9) - m.decode_step_bytes(8)
    assert per_pos == 2 * 2 * (2 * 64 + 2 * 64)                       # padded keys and values of two layers
    # past the second layer's chunk its rows start again
    assert m.decode_step_bytes(11) - m.decode_step_bytes(10) == 2 * 2 * 2 * 64 - 10 * 2 * 2 * 2 * 64
    states = 4 * (4 * 64 * 64 + 3 * 32 * 64 + 2 * 96 * 96)
    assert m.decode_step_bytes(0) > sum(a.nbytes for n, a in w.items() if n != "embed") + 2 * states
    m.close()


def test_tensors_that_do_not_fit_are_named():
    cfg, w, toks, want, _ = case("mixed")
    for name, bad in (("l0.mix.a1", None), ("l1.mix.norm", w["l1.mix.norm"][:-1]), ("l2.mix.vmix", None),
                      ("l0.mix.k.conv", w["l0.mix.k.conv"][:, :-1]), ("head", None), ("l3.norm1", None)):
        ww = {k: v for k, v in w.items() if k != name}
        if bad is not None:
            ww[name] = bad
        with pytest.raises(capi.VklError) as e:
            M.CausalModel.create(cfg, ww, None, 40)
        assert name in str(e.value)
    odd = config([attention(4, 2, 32, v_mix=True), attention(4, 4, 32, v_mix=True)], 50, 64)
    with pytest.raises(capi.VklError) as e:                          # mixed values of other sizes
        M.CausalModel.create(odd, weights(odd), None, 40)
    assert "mix values" in str(e.value)


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
    for step, rows in ((1, [52, 50]), (2, [53]), (9, [6])):
        check(np.fromfile(out / ("%d.f32" % step), "<f4").reshape(len(rows), -1), want[rows], dtype, 2)


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
