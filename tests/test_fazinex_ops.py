"""The operators of decoder stacks (include/vkl_stack.h) one by one against
float64 numpy."""
import ctypes as C

import numpy as np
import pytest

from tests import fazinex_ref as R
from tests.fazinex_util import bf16_bits, bf16_values
from vkllama_amd import capi, stack as K

pytestmark = pytest.mark.gpu
F32, BF16 = K.F32, K.BF16


def host(a, typ):
    """(array as stored, its values)"""
    if typ == F32:
        a = np.ascontiguousarray(a, np.float32)
        return a, a.astype(np.float64)
    b = bf16_bits(a)
    return b, bf16_values(b).astype(np.float64)


def read(buf, typ, shape):
    if typ == F32:
        return buf.read(np.float32, shape).astype(np.float64)
    return bf16_values(buf.read(np.uint16, shape)).astype(np.float64)


def tol(typ):
    return 2e-6 if typ == F32 else 8e-3


@pytest.mark.parametrize("xtype", [F32, BF16])
@pytest.mark.parametrize("M,N,K_", [(1, 40, 64), (2, 133, 128), (17, 1000, 320), (64, 264, 1024), (129, 136, 64),
                                    (300, 520, 2112)])
def test_project_with_segments(dev, rng, xtype, M, N, K_):
    """Columns in segments with padding between them: plain, squared relu,
    residual and soft-capped ones, in both output types; nothing is written
    beyond a segment."""
    xs = K_ + 64
    x, xv = host(rng.standard_normal((M, xs)), xtype)
    w, wv = host(rng.standard_normal((N, K_)) / np.sqrt(K_), BF16)
    full = xv[:, :K_] @ wv.T
    cut = (N // 3) // 8 * 8
    n0, n1 = cut - 3, N - cut                       # three columns of padding end the first segment
    y0 = dev.upload(np.full((M, n0 + 5), 7.0, np.float32))
    ot = BF16 if xtype == BF16 else F32
    y1 = dev.upload(np.zeros((M, n1), np.float32))
    res = rng.standard_normal((M, n0 + 5)).astype(np.float32)
    dr, dx, dw = dev.upload(res), dev.upload(x), dev.upload(w)
    segs = K.segments([(0, n0, y0.ptr, n0 + 5, F32, 0, dr.ptr, 0.0), (cut, n1, y1.ptr, n1, ot, 2, None, 0.0)])
    capi.check(K.lib().vkl_project_bf16w(dx.ptr, xtype, xs, dw.ptr, M, N, K_, segs, 2, dev.stream))
    got = y0.read(np.float32, (M, n0 + 5)).astype(np.float64)
    assert np.all(got[:, n0:] == 7.0)
    scale = np.abs(full).max()
    assert np.abs(got[:, :n0] - (full[:, :n0] + res[:, :n0])).max() < 4e-6 * scale * max(1, K_ / 256)
    want = np.square(np.maximum(full[:, cut:], 0))
    assert np.abs(read(y1, ot, (M, n1)) - want).max() < tol(ot) * np.square(scale)
    y2 = dev.alloc(M * N * 4)
    segs = K.segments([(0, N, y2.ptr, N, F32, 0, None, 0.7)])
    capi.check(K.lib().vkl_project_bf16w(dx.ptr, xtype, xs, dw.ptr, M, N, K_, segs, 1, dev.stream))
    assert np.abs(y2.read(np.float32, (M, N)) - R.softcap(full, 0.7)).max() < 5e-6


def test_embed_and_norms(dev, rng):
    W, Wp, V = 200, 256, 50
    tab = np.zeros((V, Wp), np.uint16)
    tab[:, :W] = bf16_bits(rng.standard_normal((V, W)))
    wn = rng.uniform(0.5, 1.5, W).astype(np.float32)
    toks = np.array([3, 49, 0, 3, 77], np.uint32)                 # 77 lies outside the table: row 0
    dt, dn, dk = dev.upload(tab), dev.upload(wn), dev.upload(toks)
    out = dev.upload(np.zeros((5, Wp), np.float32))
    capi.check(K.lib().vkl_embed_norm_bf16(dt.ptr, V, Wp, W, dk.ptr, 5, dn.ptr, 1e-3, out.ptr, Wp, dev.stream))
    vals = bf16_values(tab[[3, 49, 0, 3, 0], :W])
    want = R.rms_norm(vals, wn, 1e-3)
    got = out.read(np.float32, (5, Wp))
    assert np.abs(got[:, :W] - want).max() < 2e-6 and not got[:, W:].any()
    rows = dev.upload(np.array([4, 1], np.uint32))
    for typ in (F32, BF16):
        h = dev.upload(np.full(2 * Wp, 0x7fc0, np.uint32))        # (padding must become zero)
        capi.check(K.lib().vkl_rmsnorm_f32(out.ptr, Wp, rows.ptr, 2, W, dn.ptr, 0.5, h.ptr, typ, Wp, Wp, dev.stream))
        g = read(h, typ, (2, Wp))
        w2 = R.rms_norm(got[[4, 1], :W], wn, 0.5)
        assert np.abs(g[:, :W] - w2).max() < tol(typ) * np.abs(w2).max() and not g[:, W:].any()


def scores_that_stand_out(rng, S, L, H, G, D, targets):
    """q, k such that query s of every head scores one chosen key by far the
    highest: keys are random unit rows, a query is its target key scaled up"""
    k = rng.standard_normal((L, G, D))
    k /= np.linalg.norm(k, axis=2, keepdims=True)
    q = np.empty((S, H, D))
    for h in range(H):
        q[:, h] = k[targets[h % len(targets)], h // (H // G)] * 40.0
    return q, k


def edge_targets(S, L):
    """for every query a key it sees, at places where a kernel changes tile, lane
    group, split or portion: far ends, multiples of 16, 32, 64, 128 and their
    neighbours, the query itself"""
    pos = np.arange(L - S, L)
    edges = np.array([0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 255, 256, 511, 512, 1023, 1024])
    out = []
    for shift in range(4):
        t = edges[(np.arange(S) * 4 + shift) % len(edges)]
        t = np.where(t <= pos, t, np.maximum(pos - shift, 0))
        out.append(t)
    return out


@pytest.mark.parametrize("ctype", [F32, BF16])
@pytest.mark.parametrize("H,G,D,S,L", [(3, 3, 32, 1, 1), (8, 1, 32, 5, 70), (6, 2, 64, 1, 300), (12, 2, 96, 2, 129),
                                       (7, 7, 128, 3, 257), (8, 1, 160, 1, 1100), (5, 1, 256, 4, 64), (9, 1, 512, 1, 65),
                                       (4, 2, 1024, 2, 150), (8, 1, 128, 1, 4099), (2, 1, 32, 1, 2048),
                                       (33, 1, 448, 1, 900), (40, 1, 320, 2, 130), (32, 1, 512, 1, 4500), (10, 5, 384, 1, 640),
                                       (70, 2, 192, 1, 333), (4, 4, 224, 2, 200), (6, 3, 288, 1, 90)])
def test_row_attention(dev, rng, ctype, H, G, D, S, L):
    """Keys that are values, with keys planted at split and lane edges; the row
    after the last visible one holds values that would show."""
    q, k = scores_that_stand_out(rng, S, L, H, G, D, edge_targets(S, L))
    k[..., -1] += 0.01 * np.arange(L)[:, None] / L                # (rows differ in a value that is no part of the match)
    rows = np.concatenate([k, np.full((1, G, D), 1e4)])           # a row no query may see
    kb, kv = host(rows.reshape(L + 1, G * D), ctype)
    qb, qv = host(q.reshape(S, H * D), F32)
    kv = kv[:L].reshape(L, G, D)
    coef, every = 0.3, 40
    dq, dk = dev.upload(qb), dev.upload(kb)
    out = dev.alloc(S * H * D * 4)
    n = K.lib().vkl_attn_rows_scratch_bytes(ctype, H, G, D, S)
    scratch = dev.alloc(n)
    scratch.zero()
    want = np.zeros((S, H, D))
    for h in range(H):
        for s in range(S):
            p = L - S + s
            f = 0.5 * R.query_temperature(p, coef, every)
            want[s, h] = R.softmax(kv[:p + 1, h // (H // G)] @ qv.reshape(S, H, D)[s, h] * f) @ kv[:p + 1, h // (H // G)]
    for _ in range(3):                                            # the counters are left as they were found
        capi.check(K.lib().vkl_attn_rows(dq.ptr, F32, H * D, dk.ptr, ctype, G * D, H, G, D, S, L - S, 0.5, coef, every,
                                         out.ptr, F32, H * D, scratch.ptr, dev.stream))
        got = out.read(np.float32, (S, H, D))
        # (bf16 rows that several heads share: operands rounded to bf16)
        bound = 1.5e-2 if ctype == BF16 and H > G else 3e-5
        assert np.abs(got - want).max() < bound * np.abs(want).max(), np.abs(got - want).max()


@pytest.mark.parametrize("H,G,D,S,L", [(4, 4, 32, 1, 1), (8, 1, 64, 130, 130), (6, 2, 96, 200, 329), (4, 1, 128, 64, 1100),
                                       (3, 3, 160, 33, 97), (2, 1, 192, 129, 129), (2, 2, 224, 17, 80), (8, 4, 256, 140, 270)])
@pytest.mark.parametrize("gated", [False, True])
def test_prompt_attention_bf16(dev, rng, H, G, D, S, L, gated):
    q, k = scores_that_stand_out(rng, S, L, H, G, D, edge_targets(S, L))
    v = rng.standard_normal((L, G, D))
    (qb, qv), (kb, kv), (vb, vv) = host(q, BF16), host(k, BF16), host(v, BF16)
    g = rng.standard_normal((S, H + 3)).astype(np.float32)
    coef, every, scale = 0.2, 64, 0.4
    dq, dk, dv, dg = dev.upload(qb), dev.upload(kb), dev.upload(vb), dev.upload(g)
    out = dev.alloc(S * H * D * 2)
    capi.check(K.lib().vkl_attn_prefill_causal_bf16(dq.ptr, dk.ptr, dv.ptr, H, G, S, L, D, H * D, G * D, G * D, scale,
                                                    coef, every, dg.ptr if gated else None, H + 3, out.ptr, H * D,
                                                    dev.stream))
    got = read(out, BF16, (S, H, D))
    want = np.zeros((S, H, D))
    for s in range(S):
        p = L - S + s
        f = scale * R.query_temperature(p, coef, every)
        for h in range(H):
            kk, vh = kv[:p + 1, h // (H // G)], vv[:p + 1, h // (H // G)]
            want[s, h] = R.softmax(kk @ qv[s, h] * f) @ vh * (R.sigmoid(g[s, h].astype(np.float64)) if gated else 1.0)
    assert np.abs(got - want).max() < 1.2e-2 * np.abs(want).max(), np.abs(got - want).max()


@pytest.mark.parametrize("xtype", [F32, BF16])
@pytest.mark.parametrize("H,R_,K_,S", [(3, 5, 32, 1), (4, 96, 64, 3), (7, 130, 96, 2), (2, 512, 128, 1), (5, 33, 224, 16),
                                       (3, 64, 1024, 2)])
def test_head_matvec(dev, rng, xtype, H, R_, K_, S):
    w, wv = host(rng.standard_normal((H, R_, K_)) / np.sqrt(K_), BF16)
    x, xv = host(rng.standard_normal((S, H, K_)), xtype)
    g = rng.standard_normal((S, H)).astype(np.float32)
    dw, dx, dg = dev.upload(w), dev.upload(x), dev.upload(g)
    want = np.einsum("hrk,shk->shr", wv, xv)
    for gate in (False, True):
        y = dev.alloc(S * H * R_ * 4)
        capi.check(K.lib().vkl_head_matvec(dw.ptr, H, R_, K_, dx.ptr, xtype, H * K_, K_, y.ptr, F32, H * R_, R_,
                                           dg.ptr if gate else None, H, S, dev.stream))
        ref = want * R.sigmoid(g.astype(np.float64))[:, :, None] if gate else want
        assert np.abs(y.read(np.float32, (S, H, R_)) - ref).max() < 3e-6 * np.abs(ref).max()


def test_bad_shapes_are_refused(dev):
    b = dev.alloc(1 << 16)
    seg = K.segments([(0, 8, b.ptr, 8, F32, 0, None, 0.0)])
    lib = K.lib()
    assert lib.vkl_project_bf16w(b.ptr, BF16, 96, b.ptr, 1, 8, 96, seg, 1, dev.stream) == 1      # K not a multiple of 64
    late = K.segments([(4, 4, b.ptr, 8, F32, 0, None, 0.0)])
    assert lib.vkl_project_bf16w(b.ptr, BF16, 64, b.ptr, 1, 8, 64, late, 1, dev.stream) == 1     # a segment off its grid
    assert lib.vkl_attn_rows(b.ptr, F32, 48, b.ptr, F32, 48, 1, 1, 48, 1, 0, 1.0, 0.0, 1, b.ptr, F32, 48, b.ptr,
                             dev.stream) == 1
    assert lib.vkl_attn_rows(b.ptr, F32, 96, b.ptr, F32, 64, 3, 2, 32, 1, 0, 1.0, 0.0, 1, b.ptr, F32, 96, b.ptr,
                             dev.stream) == 1
    assert lib.vkl_attn_prefill_causal_bf16(b.ptr, b.ptr, b.ptr, 1, 1, 2, 1, 32, 32, 32, 32, 1.0, 0.0, 1, None, 0, b.ptr,
                                            32, dev.stream) == 1
    assert lib.vkl_attn_prefill_causal_bf16(b.ptr, b.ptr, b.ptr, 1, 1, 1, 1, 288, 288, 288, 288, 1.0, 0.0, 1, None, 0,
                                            b.ptr, 288, dev.stream) == 1
    assert lib.vkl_stack_step(None, None, 0, None, None, dev.stream) == 1
    assert C.sizeof(K.OutSeg) == 48
