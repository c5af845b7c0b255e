"""The operators of the Fuzuvik layers (include/vkl_stack.h) one by one against
the plain implementation in float64."""
import numpy as np
import pytest

from tests import fuzuvik_ref as R
from tests.test_fazinex_ops import BF16, F32, edge_targets, host, read, tol
from vkllama_amd import capi, stack as K

pytestmark = pytest.mark.gpu


def ok(rc):
    capi.check(rc)


# ---- queries, keys, values -----------------------------------------------------
@pytest.mark.parametrize("typ", [F32, BF16])
@pytest.mark.parametrize("H,G,dim,n,rot,S,pos0", [(4, 2, 64, 48, 32, 5, 0), (6, 3, 32, 32, 32, 70, 1000), (3, 1, 96, 80, 22, 3, 7),
                                                  (5, 5, 128, 128, 16, 1, 120000), (2, 1, 256, 200, 200, 9, 63),
                                                  (2, 2, 288, 270, 64, 2, 5), (3, 3, 64, 64, 0, 4, 2)])
def test_prepare_rotates_norms_and_mixes(dev, rng, typ, H, G, dim, n, rot, S, pos0):
    """Against the plain functions, in place and into other rows, on the vector
    path and off it; rows around the written ones stay."""
    f = R.frequencies({"dims": rot, "base": 7e4, "scaling": {"factor": 5.0, "low": 0.7, "high": 3.0, "original": 500}}) \
        if rot else np.empty(0)
    q = np.zeros((S, H, dim)); k = np.zeros((S, G, dim)); v = rng.standard_normal((S, G, dim))
    q[..., :n], k[..., :n] = rng.standard_normal((S, H, n)) * 3, rng.standard_normal((S, G, n))
    first = rng.standard_normal((S, G, dim))
    (qb, qv), (kb, kv), (vb, vv), (fb, fv) = host(q, typ), host(k, typ), host(v, typ), host(first, typ)
    wq = np.stack([R.rotate(qv[s, :, :n], pos0 + s, f) for s in range(S)])
    wk = np.stack([R.rotate(kv[s, :, :n], pos0 + s, f) for s in range(S)])
    wq, wk, wv = R.rms(wq, 1e-3), R.rms(wk, 1e-3), 0.7 * vv + 0.3 * fv
    rows = S + 2                                                   # a row before and one after
    es = 4 if typ == F32 else 2

    def cache(a):                                                  # device rows, and the address of position 0
        z = np.full((rows, G * dim), 3, a.dtype)
        z[1:-1] = a.reshape(S, -1)
        d = dev.upload(z)
        return d, d.ptr.value - (pos0 - 1) * G * dim * es if hasattr(d.ptr, "value") else d.ptr - (pos0 - 1) * G * dim * es
    dq, dfreq = dev.upload(qb), dev.upload(f if rot else np.zeros(1))
    (dk, k0), (dv, v0), (df, f0) = cache(kb), cache(vb), cache(fb)
    p = K.AttnRowsPrep(H, G, dim, n, len(f), dfreq.ptr, 1e-3, dq.ptr, H * dim, dq.ptr, H * dim, typ, typ,
                       k0 + pos0 * G * dim * es, v0 + pos0 * G * dim * es, G * dim, typ, k0, v0, f0, dim, 0.3, typ)
    ok(K.lib().vkl_attn_prepare(p, S, pos0, dev.stream))
    got = read(dq, typ, (S, H, dim))
    t = tol(typ) * 4
    assert np.abs(got[..., :n] - wq).max() < t * np.abs(wq).max() and not got[..., n:].any()
    gk, gv = read(dk, typ, (rows, G, dim)), read(dv, typ, (rows, G, dim))
    assert np.abs(gk[1:-1, :, :n] - wk).max() < t * np.abs(wk).max() and not gk[1:-1, :, n:].any()
    assert np.abs(gv[1:-1] - wv).max() < t * np.abs(wv).max()
    assert len(np.unique(gk[[0, -1]])) == 1 and len(np.unique(gv[[0, -1]])) == 1


def chunk_case(rng, S, L, H, G, D, size, typ):
    """Queries that each pick out one visible key - chunk edges among them - next to
    hidden keys that would win by far: the one before the chunk's start and the one
    after the query."""
    k = rng.standard_normal((L + 1, G, D))
    k /= np.linalg.norm(k, axis=2, keepdims=True)
    v = rng.standard_normal((L + 1, G, D))
    v[L] = 50.0                                                    # no query may see it
    tg = edge_targets(S, L)
    q = np.empty((S, H, D))
    for s in range(S):
        p = L - S + s
        lo = p // size * size if size else 0
        for h in range(H):
            t = max(lo, min(p, [lo, p, lo + 1][h % 4] if h % 4 < 3 else int(tg[0][s])))
            hidden = k[max(lo - 1, 0), h // (H // G)] + k[min(p + 1, L), h // (H // G)]
            q[s, h] = k[t, h // (H // G)] * 3.0 + (hidden * 9.0 if lo else 0.0)
    q[0] = 0.01 * q[0]                                             # scores near the sink's
    k[L] = k[L] * 30
    return host(q, typ), host(k, typ), host(v, typ)


def plain_rows(qv, kv, vv, scale, size, sink, S, L):
    H, G = qv.shape[1], kv.shape[1]
    out = np.zeros((S, H, vv.shape[2]))
    for s in range(S):
        p = L - S + s
        lo = p // size * size if size else 0
        for h in range(H):
            sc = kv[lo:p + 1, h // (H // G)] @ qv[s, h] * scale
            if sink:
                w = R.sink_softmax(sc)
            else:
                w = np.exp(sc - sc.max())
                w /= w.sum()
            out[s, h] = w @ vv[lo:p + 1, h // (H // G)]
    return out


@pytest.mark.parametrize("ctype", [F32, BF16])
@pytest.mark.parametrize("H,G,D,S,L,size,sink", [(4, 2, 32, 1, 1, 5, 1), (8, 1, 64, 3, 130, 64, 1), (6, 2, 96, 4, 300, 97, 1),
                                                 (4, 4, 128, 2, 1025, 1024, 1), (8, 2, 128, 1, 3000, 0, 1), (5, 1, 256, 2, 77, 33, 0),
                                                 (12, 3, 64, 2, 2500, 2400, 1), (3, 3, 288, 5, 41, 20, 1), (16, 1, 64, 1, 900, 0, 0),
                                                 (2, 1, 160, 40, 40, 1, 1), (9, 1, 512, 1, 200, 150, 1)])
def test_row_attention_with_chunks_and_sink(dev, rng, ctype, H, G, D, S, L, size, sink):
    (qb, qv), (kb, kv), (vb, vv) = chunk_case(rng, S, L, H, G, D, size, ctype)
    q32, qv = host(qv, F32)
    want = plain_rows(qv, kv, vv, 0.8, size, sink, S, L)
    dq, dk, dv = dev.upload(q32), dev.upload(kb.reshape(L + 1, -1)), dev.upload(vb.reshape(L + 1, -1))
    out = dev.alloc(S * H * D * 4)
    scratch = dev.alloc(K.lib().vkl_attn_kv_rows_scratch_bytes(ctype, H, G, D, S))
    scratch.zero()
    for _ in range(3):                                             # the counters are left as they were found
        ok(K.lib().vkl_attn_kv_rows(dq.ptr, F32, H * D, dk.ptr, dv.ptr, ctype, G * D, H, G, D, S, L - S, 0.8, size, sink,
                                    out.ptr, F32, H * D, scratch.ptr, dev.stream))
        got = out.read(np.float32, (S, H, D))
        assert np.abs(got - want).max() < 3e-5 * np.abs(want).max(), np.abs(got - want).max()


@pytest.mark.parametrize("H,G,D,S,L,size,sink", [(4, 4, 32, 1, 1, 1, 1), (8, 2, 64, 200, 200, 50, 1), (6, 2, 96, 150, 400, 64, 1),
                                                 (4, 1, 128, 300, 300, 0, 1), (8, 8, 128, 130, 1100, 1050, 1), (3, 3, 160, 70, 97, 96, 0),
                                                 (2, 1, 256, 140, 270, 129, 1), (2, 2, 64, 260, 700, 3, 1), (4, 2, 64, 128, 640, 128, 0),
                                                 (2, 1, 64, 100, 333, 200, 0)])
def test_prompt_attention_with_chunks_and_sink(dev, rng, H, G, D, S, L, size, sink):
    (qb, qv), (kb, kv), (vb, vv) = chunk_case(rng, S, L, H, G, D, size, BF16)
    want = plain_rows(qv, kv, vv, 0.8, size, sink, S, L)
    dq, dk, dv = dev.upload(qb), dev.upload(kb), dev.upload(vb)
    out = dev.alloc(S * H * D * 2)
    ok(K.lib().vkl_attn_prefill_chunked_bf16(dq.ptr, dk.ptr, dv.ptr, H, G, S, L, D, H * D, G * D, G * D, 0.8, size, sink,
                                             out.ptr, H * D, dev.stream))
    got = read(out, BF16, (S, H, D))
    assert np.abs(got - want).max() < 1.2e-2 * np.abs(want).max(), np.abs(got - want).max()


# ---- recurrences -----------------------------------------------------------------
@pytest.mark.parametrize("typ", [F32, BF16])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("cuts", [[40], [1] * 12, [2, 3, 2, 9, 1, 5], [17, 1, 4]])
def test_short_conv_over_portions(dev, rng, typ, taps, cuts):
    n, T = 24, sum(cuts)
    x, xv = host(rng.standard_normal((T, n)), typ)
    w = rng.standard_normal((n, taps))
    w[:, 0] += 2.0                                                  # the oldest input counts
    want = R.silu(R.short_conv(xv, w.astype(np.float32).astype(np.float64)))
    dw = dev.upload(np.ascontiguousarray(w.T, np.float32))
    ring = dev.upload(np.full((taps, n), 1e6, np.float32))          # what another sequence left
    at = 0
    for S in cuts:
        dx, out = dev.upload(x[at:at + S]), dev.alloc(S * n * 4)
        ok(K.lib().vkl_short_conv_silu(dx.ptr, typ, n, dw.ptr, n, taps, ring.ptr, at, S, out.ptr, n, dev.stream))
        assert np.abs(read(out, typ, (S, n)) - want[at:at + S]).max() < tol(typ) * np.abs(want).max(), at
        at += S


def recur_case(rng, typ, T, H, rep, dim, vdim, delta, n=None, strength=(-4.0, 1.5)):
    G, n = H // rep, n or dim
    q, k, v = np.zeros((T, G, dim)), np.zeros((T, G, dim)), rng.standard_normal((T, H, vdim))
    q[..., :n], k[..., :n] = rng.standard_normal((T, G, n)), rng.standard_normal((T, G, n))
    c = {"q": host(q, typ), "k": host(k, typ), "v": host(v, typ)}
    if delta:
        c["z"] = rng.uniform(-4, 2, (T, H, dim)).astype(np.float32)
        c["b"] = rng.standard_normal((T, H)).astype(np.float32)
        c["dt"] = rng.uniform(-2, 1, (H, dim)).astype(np.float32)
        c["rate"] = np.exp(rng.uniform(*strength, H)).astype(np.float32)
    else:
        c["decay"] = np.array(([1.0, 0.0, 0.5, 0.97, 0.999, 1e-3] * H)[:H])
        c["log"] = np.maximum(np.log(np.maximum(c["decay"], 1e-300)), -1e4).astype(np.float32)
    return c


def recur_plain(c, H, rep, n, delta):
    q, k, v = (np.repeat(c[x][1], rep if x != "v" else 1, axis=1) for x in "qkv")
    if not delta:
        return R.decayed_sums(q, k, v, c["decay"]) * 0.25
    q, k = (x / np.sqrt((x * x).sum(-1, keepdims=True) + R.UNIT_EPS) for x in (q, k))
    z = c["z"].astype(np.float64) + c["dt"].astype(np.float64)
    g = np.exp(-c["rate"].astype(np.float64)[None, :, None] * R.softplus(z))
    return R.delta_rule(q * 0.25, k, v, g, R.sigmoid(c["b"].astype(np.float64)))


def recur_run(dev, c, typ, H, rep, dim, vdim, cuts, form, delta, pieces=0):
    T, G = sum(cuts), H // rep
    state = dev.upload(np.full((H, dim, vdim), 1e5, np.float32))    # what another sequence left
    keep = {x: dev.upload(c[x]) for x in ("dt", "rate", "log") if x in c}
    out, at = [], 0
    for S in cuts:
        d = {x: dev.upload((c[x][0] if x in "qkv" else c[x])[at:at + S]) for x in "qkvzb" if x in c}
        y = dev.alloc(S * H * vdim * 4)
        a = K.RecurrenceArgs()
        a.H, a.rep, a.dim, a.vdim, a.type, a.qscale = H, rep, dim, vdim, typ, 0.25
        a.q, a.k, a.v, a.qs, a.ks, a.vs = d["q"].ptr, d["k"].ptr, d["v"].ptr, G * dim, G * dim, H * vdim
        a.state, a.out, a.os = state.ptr, y.ptr, H * vdim
        if delta:
            a.z, a.zs, a.b, a.bs, a.unit_eps = d["z"].ptr, H * dim, d["b"].ptr, H, R.UNIT_EPS
            a.dt_bias, a.rate = keep["dt"].ptr, keep["rate"].ptr
        else:
            a.log_decay = keep["log"].ptr
        nb = K.lib().vkl_recurrence_scratch_bytes(a, pieces or S)
        scratch = dev.alloc(max(nb, 16))
        ok(K.lib().vkl_recurrence(a, S, at, form, scratch.ptr if nb else None, nb, dev.stream))
        out.append(y.read(np.float32, (S, H, vdim)))
        at += S
    return np.concatenate(out).astype(np.float64)


SHAPES = [(4, 2, 32, 64, 150), (3, 1, 64, 32, 64), (2, 1, 128, 96, 131), (4, 4, 96, 160, 90), (1, 1, 32, 256, 65)]


@pytest.mark.parametrize("typ", [F32, BF16])
@pytest.mark.parametrize("delta", [True, False])
@pytest.mark.parametrize("H,rep,dim,vdim,T", SHAPES)
def test_recurrences_in_both_forms_and_any_portions(dev, rng, typ, delta, H, rep, dim, vdim, T):
    if not delta:
        rep = 1
    c = recur_case(rng, typ, T, H, rep, dim, vdim, delta, n=dim - 3)
    want = recur_plain(c, H, rep, dim - 3, delta)
    for cuts in ([T], [2, 1, 30, 2, T - 35]):
        for form in (K.RECUR_TOKENS, K.RECUR_CHUNKS, K.RECUR_AUTO):
            got = recur_run(dev, c, typ, H, rep, dim, vdim, cuts, form, delta)
            err = np.abs(got - want).max(axis=(0, 2)) / np.abs(want).max(axis=(0, 2))
            assert err.max() < 2e-5, (cuts, form, err)
    # in pieces of one chunk, for want of scratch memory
    got = recur_run(dev, c, typ, H, rep, dim, vdim, [T], K.RECUR_CHUNKS, delta, pieces=64)
    assert np.abs(got - want).max() < 2e-5 * np.abs(want).max()


@pytest.mark.parametrize("strength", [(-12.0, -9.0), (2.0, 3.0), (5.0, 7.0), (-12.0, 7.0)])
def test_delta_rule_with_decays_from_none_to_total(dev, rng, strength):
    """Blocks whose decay leaves the range of a float are formed pair by pair; a
    channel that hardly decays remembers the first token, one that decays at once
    the last."""
    H, dim, vdim, T = 4, 64, 32, 200
    c = recur_case(rng, F32, T, H, 1, dim, vdim, True, strength=strength)
    c["dt"][:, ::2] = -9.0                                          # strong and weak channels side by side
    c["z"][60:64] = 30.0                                            # a burst at the end of a chunk
    want = recur_plain(c, H, 1, dim, True)
    for form in (K.RECUR_TOKENS, K.RECUR_CHUNKS):
        got = recur_run(dev, c, F32, H, 1, dim, vdim, [T], form, True)
        assert np.isfinite(got).all() and np.abs(got - want).max() < 3e-5 * np.abs(want).max(), form


@pytest.mark.parametrize("dim", [160, 256])
def test_recurrences_of_wide_heads(dev, rng, dim):
    for delta in (True, False):
        c = recur_case(rng, BF16, 70, 2, 1, dim, 64, delta)
        want = recur_plain(c, 2, 1, dim, delta)
        got = recur_run(dev, c, BF16, 2, 1, dim, 64, [40, 30], K.RECUR_AUTO, delta)
        assert np.abs(got - want).max() < 2e-5 * np.abs(want).max()


def test_a_state_holds_far_tokens(dev, rng):
    """One key among hundreds, asked for long after: with a decay of one nothing of
    it may be lost at a chunk's edge."""
    T, dim, vdim = 700, 64, 32
    for hit in (0, 62, 63, 64, 65, 127, 128, 511):
        c = recur_case(rng, F32, T, 1, 1, dim, vdim, False)
        q, k, v = (c[x][1] * s for x, s in zip("qkv", (0.0, 0.0, 1.0)))
        k[hit, 0, 5], q[-1, 0, 5], q[min(hit + 1, T - 1), 0, 5] = 2.0, 1.0, 1.0
        for x, a in zip("qkv", (q, k, v)):
            c[x] = host(a, F32)
        got = recur_run(dev, c, F32, 1, 1, dim, vdim, [300, 2, 397, 1], K.RECUR_AUTO, False)
        assert np.allclose(got[-1, 0], 0.5 * v[hit, 0], rtol=1e-5) and np.allclose(got[hit + 1, 0], 0.5 * v[hit, 0], rtol=1e-5)


@pytest.mark.parametrize("typ", [F32, BF16])
@pytest.mark.parametrize("dim,r,T", [(32, 64, 40), (128, 128, 150), (96, 192, 65)])
def test_decays_of_low_rank_inside_the_chunked_form(dev, rng, typ, dim, r, T):
    H, vdim = 3, 32
    c = recur_case(rng, typ, T, H, 1, dim, vdim, True)
    a1, av = host(rng.standard_normal((T, r)), typ)
    w, wv = host(rng.standard_normal((H * dim, r)) / np.sqrt(r), BF16)
    c["z"] = (av @ wv.T).reshape(T, H, dim)
    want = recur_plain(c, H, 1, dim, True)
    d = {x: dev.upload(c[x][0]) for x in "qkv"}
    db, dt, rate, da, dw = (dev.upload(x) for x in (c["b"], c["dt"], c["rate"], a1, w))
    state, out = dev.alloc(H * dim * vdim * 4), dev.alloc(T * H * vdim * 4)
    a = K.RecurrenceArgs(H, 1, dim, vdim, d["q"].ptr, d["k"].ptr, d["v"].ptr, typ, H * dim, H * dim, H * vdim, 0.25, None,
                         None, 0, da.ptr, r, dw.ptr, r, db.ptr, H, dt.ptr, rate.ptr, R.UNIT_EPS, state.ptr, out.ptr,
                         H * vdim)
    n = K.lib().vkl_recurrence_scratch_bytes(a, T)
    scratch = dev.alloc(n)
    assert K.lib().vkl_recurrence_chunked(a, T) == 1
    ok(K.lib().vkl_recurrence(a, T, 0, K.RECUR_AUTO, scratch.ptr, n, dev.stream))
    assert np.abs(out.read(np.float32, (T, H, vdim)) - want).max() < 3e-5 * np.abs(want).max()
    assert K.lib().vkl_recurrence(a, T, 0, K.RECUR_TOKENS, scratch.ptr, n, dev.stream) == 1   # needs z


@pytest.mark.parametrize("typ", [F32, BF16])
@pytest.mark.parametrize("groups,gw,n,S", [(4, 32, 24, 9), (3, 96, 96, 70), (1, 320, 250, 33), (2, 256, 256, 1), (1, 4096, 4096, 3)])
def test_gated_norms(dev, rng, typ, groups, gw, n, S):
    x = np.zeros((S, groups, gw), np.float32)
    x[..., :n] = rng.standard_normal((S, groups, n))
    w = rng.uniform(0.5, 1.5, (groups if groups == 1 else 1, gw)).astype(np.float32)
    g, gv = host(rng.standard_normal((S, groups, gw)), typ)
    dx, dw, dg, out = dev.upload(x), dev.upload(w), dev.upload(g), dev.alloc(S * groups * gw * 4)
    ok(K.lib().vkl_gated_norm(dx.ptr, groups * gw, groups, gw, n, dw.ptr, 1e-2, dg.ptr, groups * gw, typ, S, out.ptr,
                              groups * gw, dev.stream))
    norm = np.zeros(x.shape)
    norm[..., :n] = R.rms(x[..., :n], 1e-2)
    want = norm * w * R.sigmoid(gv)
    assert np.abs(read(out, typ, x.shape) - want).max() < tol(typ) * 2 * np.abs(want).max()
    if gw > 256 or gw % 32:
        return
    for r in (64, 128):
        g1, g1v = host(rng.standard_normal((S, r)), typ)
        g2, g2v = host(rng.standard_normal((groups * gw, r)) / np.sqrt(r), BF16)
        d1, d2 = dev.upload(g1), dev.upload(g2)
        ok(K.lib().vkl_low_rank_gated_norm(dx.ptr, groups * gw, groups, gw, n, dw.ptr, 1e-2, d1.ptr, r, d2.ptr, r, typ, S,
                                           out.ptr, groups * gw, dev.stream))
        want = norm * w * R.sigmoid(g1v @ g2v.T).reshape(S, groups, gw)
        assert np.abs(read(out, typ, x.shape) - want).max() < tol(typ) * 2 * np.abs(want).max(), r


# ---- products and embedding -----------------------------------------------------
@pytest.mark.parametrize("typ", [F32, BF16])
def test_activations_of_products(dev, rng, typ):
    M, N, K_ = 70, 96, 128
    x, xv = host(rng.standard_normal((M, K_)), typ)
    w, wv = host(rng.standard_normal((N, K_)) / np.sqrt(K_), BF16)
    dx, dw = dev.upload(x), dev.upload(w)
    full = xv @ wv.T
    for act, fn in ((K.ACT_NONE, lambda z: z), (K.ACT_SILU, R.silu), (K.ACT_GELU, R.gelu)):
        y = dev.alloc(M * N * 4)
        seg = K.segments([(0, N, y.ptr, N, typ, act, None, 0.0)])
        ok(K.lib().vkl_project_bf16w(dx.ptr, typ, K_, dw.ptr, M, N, K_, seg, 1, dev.stream))
        want = fn(full)
        assert np.abs(read(y, typ, (M, N)) - want).max() < tol(typ) * np.abs(want).max(), act
    seg = K.segments([(0, N, dx.ptr, N, typ, 4, None, 0.0)])
    assert K.lib().vkl_project_bf16w(dx.ptr, typ, K_, dw.ptr, M, N, K_, seg, 1, dev.stream) == 1


@pytest.mark.parametrize("W,Wp", [(40, 64), (33, 64), (256, 256)])
def test_scaled_embedding(dev, rng, W, Wp):
    tab = np.zeros((9, Wp), np.uint16)
    tab[:, :W], vals = host(rng.standard_normal((9, W)), BF16)
    toks = dev.upload(np.array([8, 0, 3, 8], np.uint32))
    dt, out = dev.upload(tab), dev.upload(np.zeros((4, Wp), np.float32))
    ok(K.lib().vkl_embed_rows_bf16(dt.ptr, 9, Wp, W, toks.ptr, 4, 2.5, out.ptr, Wp, dev.stream))
    got = out.read(np.float32, (4, Wp))
    assert np.allclose(got[:, :W], vals[[8, 0, 3, 8]] * 2.5, rtol=1e-6) and not got[:, W:].any()


def test_bad_shapes_are_refused(dev):
    b, lib = dev.alloc(1 << 16), K.lib()
    a = K.RecurrenceArgs()
    a.H, a.rep, a.dim, a.vdim = 2, 1, 48, 32                        # dim off its grid
    assert lib.vkl_recurrence(a, 4, 0, 0, None, 0, dev.stream) == 1 and lib.vkl_recurrence_scratch_bytes(a, 4) == 0
    a.dim = 32
    a.q = a.k = a.v = a.state = a.out = a.log_decay = b.ptr
    a.qs = a.ks = a.vs = a.os = 64
    assert lib.vkl_recurrence(a, 64, 0, K.RECUR_CHUNKS, None, 0, dev.stream) == 1               # no scratch memory
    a.rep = 4
    assert lib.vkl_recurrence(a, 4, 0, K.RECUR_TOKENS, None, 0, dev.stream) == 1                # heads do not divide
    assert lib.vkl_short_conv_silu(b.ptr, F32, 8, b.ptr, 8, 17, b.ptr, 0, 1, b.ptr, 8, dev.stream) == 1
    assert lib.vkl_gated_norm(b.ptr, 32, 1, 32, 33, b.ptr, 1e-5, b.ptr, 32, F32, 1, b.ptr, 32, dev.stream) == 1
    p = K.AttnRowsPrep(H=1, G=1, dim=32, n=32, npair=17)
    assert lib.vkl_attn_prepare(p, 1, 0, dev.stream) == 1
    assert lib.vkl_attn_kv_rows(b.ptr, F32, 32, b.ptr, None, F32, 32, 1, 1, 32, 1, 0, 1.0, 0, 1, b.ptr, F32, 32, b.ptr,
                                dev.stream) == 1
    assert lib.vkl_attn_prefill_chunked_bf16(b.ptr, b.ptr, b.ptr, 1, 1, 1, 1, 32, 32, 32, 32, 1.0, -1, 1, b.ptr, 32,
                                             dev.stream) == 1
