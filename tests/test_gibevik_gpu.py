"""The Gibevik family (the post-norm form of the layer stack: sinusoidal positions in the embedding, grouped-query attention whose values are its raw keys with a norm per
head, a query temperature, a bias falling with the distance and an elementwise gate, latent attention without positions that may read an earlier layer's latents, dense
gated units and mixtures of squared-relu experts chosen with a correction among groups, some of them the identity) against tests/gibevik_oracle.py -- a float64
restatement that shares nothing with the product.  Every test makes its own small configuration and random bf16-representable weights, writes them as a model folder and
runs them through the C API (the engine's step function, slot cache and kernels); the operator tests call include/ntk_layers.h directly.

Error measure: rms of the difference over rms of the reference.  float32 mode is held to 2e-4 (observed ~1e-6), bfloat16 mode to 4e-2."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import gibevik_oracle as O  # noqa: E402

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": 2e-4, "bfloat16": 4e-2}
F64 = np.float64


def rel(got, ref):
    got, ref = np.asarray(got, F64), np.asarray(ref, F64)
    return float(np.sqrt(np.mean((got - ref) ** 2)) / (np.sqrt(np.mean(ref ** 2)) + 1e-30))


def row_err(got, ref):
    got, ref = np.asarray(got, F64), np.asarray(ref, F64)
    return np.sqrt(np.mean((got - ref) ** 2, axis=1)) / np.sqrt(np.mean(ref ** 2))


def make(tmp_path, cfg, seed=1, name="m", gain=1.0, change=None):
    w = O.random_weights(cfg, seed, gain)
    if change:
        change(w)
    folder = str(tmp_path / name)
    O.save_model(folder, cfg, w)
    return folder, w


def engine_for(folder, dtype="float32", ctx=512, slots=1):
    from ntransformer_amd.engine import Engine
    e = Engine()
    e.load_folder(folder, max_context=ctx, dtype=dtype, slots=slots)
    return e


def tokens_for(cfg, n, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def f32(a):
    return np.asarray(a, np.float32)


def mixed(**kw):
    """both kinds of mixer and of feed-forward, a layer that reads another one's latents across one with keys of its own (and with other heads and sizes than the layer it
    reads), a temperature that steps within the test's lengths, one layer without feed-forward"""
    return O.config([O.layer_latent(mlp=O.dense(40)), O.layer_attention(every=7, mlp=O.moe(9, 3, 12, identity=3, groups=(3, 1), shared=20)),
                     O.layer_latent(kv_from=0, heads=3, dim=10, vdim=6, mlp=O.moe(5, 2, 16)), O.layer_attention(heads=6, kv_heads=1, dim=12, coef=0),
                     O.layer_latent(kv_rank=24, mlp=O.dense())], **kw)


# the choice of experts is discontinuous: bfloat16 products may turn a close one, and the row then differs by a whole expert.  Rows are compared where the oracle's own
# choice has a margin (bfloat16 only; float32 mode is held to every row).
def clear_rows(cfg, w, toks, margin=0.02):
    """rows whose every routed choice (groups and experts) keeps a margin in the oracle, up to and with all earlier rows' influence being smooth"""
    ok = np.ones(len(toks), bool)
    real = O.route

    def probe(z, correction, top, groups=None):
        s = O.softmax(z) + correction
        if groups:
            per = len(s) // groups["count"]
            best = np.array([max(s[g * per:(g + 1) * per]) for g in range(groups["count"])])
            o = np.sort(best)[::-1]
            gap = o[groups["keep"] - 1] - o[groups["keep"]] if groups["keep"] < groups["count"] else 1.0
            kept = np.argsort(-best, kind="stable")[:groups["keep"]]
            s = np.where(np.isin(np.arange(len(s)) // per, kept), s, -np.inf)
        else:
            gap = 1.0
        o = np.sort(s)[::-1]
        if top < len(o):
            gap = min(gap, o[top - 1] - o[top])
        if gap < margin:
            ok[probe.row % len(toks)] = False
        probe.row += 1
        return real(z, correction, top, groups)

    probe.row = 0
    O.route = probe
    try:
        O.forward(cfg, w, toks)
    finally:
        O.route = real
    return ok


def close(cfg, w, toks, got, ref, dtype, at=0):
    """got / ref are rows at .. of toks"""
    if dtype == "float32":
        return rel(got, ref) < TOL[dtype] and row_err(got, ref).max() < 3 * TOL[dtype]
    ok = clear_rows(cfg, w, toks)[at:at + len(got)]
    assert ok.mean() > 0.3
    return float(np.median(row_err(got, ref)[ok])) < TOL[dtype]


# ====================================================================================================================== operators
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("V,W,pos0", [(61, 33, 0), (300, 520, 7), (17, 8, 4000), (5, 1, 3), (9, 2, 100000)])
def test_embedding_row_plus_the_position_vector(dtype, V, W, pos0):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(V)
    E = O.to_bf16(g.standard_normal((V, W)))
    toks = [int(t) for t in g.integers(0, V, 9)]
    freq = [10000.0 ** (-2.0 * i / W) for i in range((W + 1) // 2)]
    assert np.abs(Lr.embed_sinusoid(E, toks, pos0, freq, dtype=dtype) - O.embed({"embed": E}, toks, pos0)).max() < 1e-6
    assert np.abs(Lr.embed_sinusoid(E, toks, pos0, freq, 2.5, dtype=dtype) - O.embed({"embed": 2.5 * E}, toks, pos0)).max() < 2e-6


@pytest.mark.parametrize("H,G,dn,dims,halves", [(4, 2, 8, 0, 0), (8, 1, 48, 0, 0), (3, 3, 7, 0, 0), (1, 1, 1, 0, 0), (16, 4, 128, 0, 0), (2, 1, 300, 0, 0), (4, 2, 16, 12, 1), (3, 1, 10, 10, 0), (2, 2, 270, 130, 1)])
@pytest.mark.parametrize("T,pos0", [(1, 0), (1, 48), (1, 49), (5, 47), (40, 130)])
def test_norm_per_head_then_temperature_and_raw_keys_as_values(H, G, dn, dims, halves, T, pos0):
    """one loud head (a norm over the whole projection would not level it); the temperature multiplies the NORMED query and steps at position 49; values are the keys as
    they came; the same with a rotation behind the norm"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(H * 100 + dn + T)
    q, k = f32(g.standard_normal((T, H * dn)) * 3), f32(g.standard_normal((T, G * dn)) * 0.2)
    q[:, :dn] *= 20.0
    qn, kn = f32(1 + 0.3 * g.standard_normal(dn)), f32(1 + 0.3 * g.standard_normal(dn))
    eps, qt = 1e-3, {"coef": 0.7, "every": 50}
    freq = np.array([500.0 ** (-2.0 * i / dims) for i in range(dims // 2)], F64)

    def rotated(z):
        y = z.copy()
        for t in range(T):
            a = (pos0 + t) * freq
            i = np.arange(dims // 2)
            u, v = (i, i + dims // 2) if halves else (2 * i, 2 * i + 1)
            y[t][:, u], y[t][:, v] = z[t][:, u] * np.cos(a) - z[t][:, v] * np.sin(a), z[t][:, v] * np.cos(a) + z[t][:, u] * np.sin(a)
        return y

    qb, kb = f32(g.standard_normal(H * dn)), f32(g.standard_normal(G * dn))
    for bias in (False, True):
        q1, k1 = q.astype(F64) + (qb if bias else 0), k.astype(F64) + (kb if bias else 0)
        temp = np.array([O.temperature(pos0 + t, qt) for t in range(T)])[:, None, None]
        qr = rotated(O.rms(q1.reshape(T, H, dn), qn.astype(F64), eps) * temp).reshape(T, -1)
        kr = rotated(O.rms(k1.reshape(T, G, dn), kn.astype(F64), eps)).reshape(T, -1)
        kw = dict(freq=freq, dims=dims, layout=Lr.ROT_HALVES if halves else Lr.ROT_NEIGHBOURS, norm_eps=eps, head_norm=True, temp_coef=0.7, temp_every=50.0)
        if bias:
            kw.update(qb=qb, kb=kb)
        cache, gq, _ = Lr.window_prepare_ex(q, k, None, H, G, dn, dn, pos0, q_norm=qn, k_norm=kn, values_are_keys=True, **kw)
        assert rel(gq, qr) < 1e-5 and rel(cache[pos0:, :G * dn], kr) < 1e-5 and np.array_equal(cache[pos0:, G * dn:], k) and not cache[:pos0].any()
    v = f32(g.standard_normal((T, G * 5)))                                               # values of their own, and queries alone
    kw.pop("qb"), kw.pop("kb")
    cache, gq, _ = Lr.window_prepare_ex(q, k, v, H, G, dn, 5, pos0, q_norm=qn, k_norm=kn, **kw)
    assert np.array_equal(cache[pos0:, G * dn:], v)
    before = f32(g.standard_normal((pos0 + T, G * (dn + 5))))
    cache, gq2, _ = Lr.window_prepare_ex(q, None, None, H, G, dn, 5, pos0, q_norm=qn, cache=before, **kw)
    assert np.array_equal(cache, before) and np.array_equal(gq, gq2)


@pytest.mark.parametrize("H,G,dn,dv", [(4, 2, 12, 20), (3, 3, 5, 3), (6, 1, 70, 130), (1, 1, 8, 8), (8, 2, 96, 96)])
@pytest.mark.parametrize("pos0,T", [(0, 50), (330, 1), (325, 6), (60, 23), (1200, 1), (1190, 20)])
def test_attention_with_a_bias_falling_with_the_distance(H, G, dn, dv, pos0, T):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(H * 1000 + pos0)
    P = pos0 + T
    q, K, V = f32(g.standard_normal((T, H * dn))), f32(g.standard_normal((P, G * dn))), f32(g.standard_normal((P, G * dv)))
    cache = np.concatenate([K, V], axis=1)
    sl = f32([O.slope(h, H) for h in range(H)])
    gate = f32(g.standard_normal((T, H * dv)) * 2)
    scale = 1.5 / math.sqrt(dn)
    ref = O.attend(q.reshape(T, H, dn).astype(F64), K.reshape(P, G, dn).astype(F64), V.reshape(P, G, dv).astype(F64), pos0, scale, sl).reshape(T, -1)
    for split in (True, False):
        assert rel(Lr.window_attention(q, cache, H, G, 1, dn, dv, pos0, 0, scale, split=split, slopes=sl), ref) < 1e-5, split
        assert rel(Lr.window_attention(q, cache, H, G, 1, dn, dv, pos0, 0, scale, split=split, slopes=sl, gate=gate), ref * O.sigmoid(gate.astype(F64))) < 1e-5, split


def test_the_distance_bias_against_a_towering_key():
    """two keys stand out, the farther one by `lead` more: head h prefers it exactly while slope_h * (their distance) stays below the lead -- over hundreds of keys, across
    64-key steps, split and unsplit, decoded and in portions"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(8)
    H, dn, dv, P = 8, 16, 8, 900
    sl = f32([O.slope(h, H) for h in range(H)])
    d = g.standard_normal(dn)
    d /= np.linalg.norm(d)
    for near, far in ((899, 898), (870, 868), (830, 767), (640, 639), (700, 60), (64, 63), (600, 0)):
        K, V = f32(0.01 * g.standard_normal((P, dn))), f32(g.standard_normal((P, dv)))
        lead = 12.0
        K[near] = 500.0 * d
        K[far] = (500.0 + lead) * d
        q = f32(np.tile(d, (P, H)))
        cache = np.concatenate([K, V], axis=1)
        for pos0, T in ((P - 1, 1), (P - 5, 5), (P - 30, 30)):
            if pos0 < near:
                continue
            for split in (True, False):
                got = Lr.window_attention(q[pos0:], cache, H, 1, 1, dn, dv, pos0, 0, 1.0, split=split, slopes=sl).reshape(T, H, dv)
                for h in range(H):
                    gap = lead - float(sl[h]) * (near - far)
                    if float(sl[h]) * (P - 1 - near) > 400 or abs(gap) < 8:
                        continue                                                         # (the pair does not stand out, or is not decided)
                    assert np.abs(got[:, h] - V[far if gap > 0 else near]).max() < 5e-3, (near, far, pos0, h)


def test_a_far_latent_among_hundreds():
    """latent attention has no positions: one towering latent is found at any distance, across 32-row tiles and splits, in the few-token and the expanded form"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(9)
    H, dn, dv, R, P = 3, 12, 10, 40, 1300
    uk, uv = g.standard_normal((H * dn, R)) / math.sqrt(R), g.standard_normal((H * dv, R)) / math.sqrt(R)
    for tower in (0, 31, 32, 63, 64, 700, 1279):
        c = f32(g.standard_normal((P, R)))
        k, v = (c.astype(F64) @ uk.T).reshape(P, H, dn), (c.astype(F64) @ uv.T).reshape(P, H, dv)
        q = 0.05 * g.standard_normal((12, H, dn))
        c1 = c.copy()
        c1[tower] *= 6.0
        k, v = (c1.astype(F64) @ uk.T).reshape(P, H, dn), (c1.astype(F64) @ uv.T).reshape(P, H, dv)
        q[:, 1] += 8.0 * k[tower, 1] / np.linalg.norm(k[tower, 1])
        for T in (1, 5, 12):
            ref = O.attend(q[-T:], k, v, P - T, 1.0)
            qt = f32(q[-T:].reshape(T, -1))
            if T <= 8:
                lat = Lr.latent_attention(Lr.latent_fold_query(qt, uk, H, dn, 0), c1, R, 0, H, P - T, 0, 1.0)
                got = Lr.latent_unfold_value(lat, uv, H)
            else:
                got = Lr.latent_attention(qt, c1, R, 0, H, P - T, 0, 1.0, K=f32(k.reshape(P, -1)), V=f32(v.reshape(P, -1)))
            assert rel(got, ref.reshape(T, -1)) < 1e-4, (tower, T)
            assert np.abs(got.reshape(T, H, dv)[:, 1] - v[tower, 1]).max() < 2e-2 * np.abs(v[tower, 1]).max(), (tower, T)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,H,dn,R", [(1, 4, 8, 16), (8, 3, 7, 33), (2, 1, 1, 1), (3, 2, 128, 512), (5, 16, 24, 65)])
def test_query_fold_with_the_cache_rows_beside_it(dtype, T, H, dn, R):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(H + R)
    q, uk = f32(g.standard_normal((T, H * dn))), O.to_bf16(g.standard_normal((H * dn, R)))
    kv, nw = f32(g.standard_normal((T, R + 3)) * 4), f32(1 + 0.2 * g.standard_normal(R))
    cache = f32(g.standard_normal((T + 9, R + 2)))
    qf, after = Lr.latent_fold_query_prepare(q, uk, H, dn, kv, nw, 1e-4, 5, cache, dtype)
    assert rel(qf, np.einsum("thd,hdr->thr", q.reshape(T, H, dn).astype(F64), uk.reshape(H, dn, R)).reshape(T, -1)) < 1e-5
    assert rel(after[5:5 + T, :R], O.rms(kv[:, :R].astype(F64), nw.astype(F64), 1e-4)) < 1e-5
    same = np.ones(cache.shape, bool)
    same[5:5 + T, :R] = False
    assert np.array_equal(after[same], cache[same])


@pytest.mark.parametrize("E,top,groups,keep", [(6, 2, 1, 1), (15, 4, 3, 1), (12, 3, 4, 2), (130, 9, 1, 1), (255, 30, 5, 3), (1, 1, 1, 1), (64, 64, 1, 1), (8, 4, 8, 4), (200, 2, 100, 1)])
def test_router_with_a_correction(E, top, groups, keep):
    """choice scores of both signs, corrections that overturn the scores' own order, groups whose best choice score is negative, ties resolved to the lower index"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(E + top)
    n, T = 44, 12
    wr = f32(g.standard_normal((E, n)))
    for shift in (-3.0, 0.0, 2.0):
        h, corr = f32(g.standard_normal((T, n)) * 0.3), f32(g.uniform(-1, 1, E) + shift)
        ids, wts = Lr.moe_route_ex(h, wr, top, score=0, groups=groups, keep=keep, group_top=1, correction=corr)
        for t in range(T):
            want = O.route(wr.astype(F64) @ h[t].astype(F64), corr.astype(F64), top, {"count": groups, "keep": keep} if groups > 1 else None)
            assert list(ids[t]) == [e for e, _ in want], (shift, t)
            assert np.allclose(wts[t], [s for _, s in want], rtol=2e-5, atol=1e-9)
        z = f32(np.concatenate([h.astype(F64) @ wr.T.astype(F64), g.standard_normal((T, 1))], axis=1))      # the choice alone, behind a product that also formed a gate
        pids, pw, sg = Lr.moe_pick(z, E, top, groups=groups, keep=keep, correction=corr)
        assert np.array_equal(pids, ids) and np.allclose(pw, wts, rtol=1e-4, atol=1e-9) and np.allclose(sg, O.sigmoid(z[:, -1].astype(F64)), rtol=1e-6)
        assert Lr.moe_pick(z[:, :-1], E, top, groups=groups, keep=keep, correction=corr)[2] is None
    ids, wts = Lr.moe_route_ex(np.zeros((2, n), np.float32), wr, top, score=0, groups=groups, keep=keep, group_top=1, correction=np.full(E, -7.0, np.float32))
    assert list(ids[0]) == list(range(top)) and np.allclose(wts, 1.0 / E)
    y, aw = f32(g.standard_normal((T, n)) * 5), f32(1 + 0.3 * g.standard_normal(n))      # what the rows are still owed joins them first
    h2 = h.astype(F64) + O.rms(y.astype(F64), aw.astype(F64), 1e-3)
    ids, wts, hh = Lr.moe_route_ex(h, wr, top, score=0, groups=groups, keep=keep, group_top=1, correction=corr, add=(y, aw, 1e-3))
    assert rel(hh, h2) < 1e-6
    for t in range(T):
        want = O.route(wr.astype(F64) @ h2[t], corr.astype(F64), top, {"count": groups, "keep": keep} if groups > 1 else None)
        assert set(ids[t]) == {e for e, _ in want} and np.allclose(np.sort(wts[t]), np.sort([s for _, s in want]), rtol=1e-4, atol=1e-9), t


def test_squared_relu_inside_every_form_of_the_product():
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(4)
    for T, N, K in ((1, 24, 16), (8, 70, 33), (3, 4200, 264), (9, 40, 24), (70, 150, 64), (300, 260, 128), (33, 30, 7)):
        x, w = f32(g.standard_normal((T, K))), O.to_bf16(g.standard_normal((N, K)))
        for dtype, tol in (("float32", 1e-5), ("bfloat16", 1e-5 if T <= 8 else 2e-2)):
            assert rel(Lr.dense(x, w, dtype, act=Lr.ACT_RELU2), O.squared_relu(x.astype(F64) @ w.T)) < tol, (T, N, K, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,N,K", [(1, 24, 16), (3, 70, 33), (8, 4200, 264), (1, 5000, 2056), (2, 64, 4104), (1, 40, 9000), (5, 30, 16384)])
def test_few_row_products_with_the_owed_sum_inside(dtype, T, N, K):
    """x + mult * rms(y) * w on the way into a product: the product's result and the rows it leaves, alone, with a norm of the sum, and with the gated unit behind it"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(N + K)
    x, y, aw, nw = f32(g.standard_normal((T, K)) * 3), f32(g.standard_normal((T, K)) * 0.3), f32(1 + 0.3 * g.standard_normal(K)), f32(1 + 0.3 * g.standard_normal(K))
    w = O.to_bf16(g.standard_normal((N, K)) / math.sqrt(K))
    h = x.astype(F64) + 0.8 * O.rms(y.astype(F64), aw.astype(F64), 1e-3)
    add = (y, aw, 1e-3, 0.8)
    got, hh = Lr.dense(x, w, dtype, add=add)
    assert rel(got, h @ w.T) < 1e-5 and rel(hh, h) < 1e-6
    got, hh = Lr.dense(x, w, dtype, add=add, norm_w=nw, norm_eps=1e-2)
    assert rel(got, O.rms(h, nw.astype(F64), 1e-2) @ w.T) < 1e-5 and rel(hh, h) < 1e-6
    gu = h @ w.T
    got, hh = Lr.dense(x, w, dtype, add=add, glu_limit=float("inf"), glu_alpha=1.0, glu_up_offset=0.0)
    assert rel(got, O.silu(gu[:, :N // 2]) * gu[:, N // 2:]) < 1e-5 and rel(hh, h) < 1e-6
    got, hh = Lr.dense(x, w, dtype, add=add, act=Lr.ACT_RELU2)
    assert rel(got, O.squared_relu(gu)) < 1e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,n,E,ff,top,sff", [(1, 32, 4, 16, 2, 24), (8, 40, 6, 8, 3, 0), (3, 33, 5, 7, 4, 11), (2, 600, 3, 520, 3, 1032), (5, 8, 1, 8, 1, 8), (1, 2048, 9, 200, 6, 1416), (4, 24, 5, 48, 5, 3)])
def test_a_few_tokens_experts_in_two_launches(dtype, T, n, E, ff, top, sff):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(n + ff)
    h = f32(g.standard_normal((T, n)))
    up, down = O.to_bf16(g.standard_normal((E, ff, n)) / math.sqrt(n)), O.to_bf16(g.standard_normal((E, n, ff)) / math.sqrt(ff))
    su, sd = (O.to_bf16(g.standard_normal((sff, n)) / math.sqrt(n)), O.to_bf16(g.standard_normal((n, sff)) / math.sqrt(sff))) if sff else (None, None)
    sg = f32(g.uniform(0, 1, T)) if sff else None
    for identity in (0, 1, top):                                             # none, some, only identity experts
        ids = np.stack([g.permutation(E + 2)[:top] for _ in range(T)]) if identity == 1 else np.stack([g.permutation(max(E, top))[:top] % E for _ in range(T)]) + (E if identity == top else 0)
        wts = f32(g.uniform(0.1, 1, (T, top)))
        ref = np.zeros((T, n))
        for t in range(T):
            x = h[t].astype(F64)
            for e, wt in zip(ids[t], wts[t]):
                ref[t] += wt * (down[e] @ O.squared_relu(up[e] @ x) if e < E else x)
            if sff:
                ref[t] += sg[t] * (sd @ O.squared_relu(su @ x))
        assert rel(Lr.moe_few(h, ids, wts, up, down, su, sd, sg, dtype=dtype), ref) < 1e-5, identity


def test_weighted_sum_with_identity_experts():
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(6)
    for T, top, n, E in ((1, 2, 5, 3), (40, 4, 300, 6), (9, 1, 64, 1)):
        ids = g.integers(0, E + 2, (T, top))
        off, order, where = Lr.moe_group(ids, E + 2)
        d = f32(g.standard_normal((T * top, n)))
        d[off[E]:] = np.nan                                                  # rows behind the experts with matrices are never written
        h, wts = f32(g.standard_normal((T, n))), f32(g.uniform(0, 1, (T, top)))
        sh, sg = f32(g.standard_normal((T, n))), f32(g.uniform(0, 1, T))
        got = Lr.moe_sum(d, where, wts, sh, sg, ids=ids, n_experts=E, h=h)
        ref = sg[:, None].astype(F64) * sh
        for t in range(T):
            for s in range(top):
                ref[t] += wts[t, s] * (h[t] if ids[t, s] >= E else d[where[t * top + s]]).astype(F64)
        assert rel(got, ref) < 1e-6
        plain = f32(g.standard_normal((T * top, n)))
        assert rel(Lr.moe_sum(plain, None, wts), np.einsum("ts,tsn->tn", wts.astype(F64), plain.reshape(T, top, n))) < 1e-6


# ====================================================================================================================== whole models
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [60, 5])
def test_whole_prompt_with_the_stream_after_every_layer(tmp_path, dtype, n):
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=2)
    toks = tokens_for(cfg, n, seed=3)
    streams = []
    ref, _ = O.forward(cfg, w, toks, layers_out=streams)
    e = engine_for(folder, dtype)
    assert e.layer_runs == 5
    e.seq_capture(True)
    s = e.seq_acquire()
    got = e.seq_forward(s, toks)
    cap = e.seq_captured(len(toks))
    for i in range(5):
        assert close(cfg, w, toks, cap[i], streams[i], dtype), i
    assert close(cfg, w, toks, got, ref, dtype)
    e.seq_capture(False)
    e.seq_release(s)
    s = e.seq_acquire()
    some = e.seq_forward(s, toks, want=[0, 3, n - 1])                        # wanted places only
    assert rel(some, got[[0, 3, n - 1]]) < (1e-5 if dtype == "float32" else TOL[dtype])
    e.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prefill_against_token_by_token_and_portions(tmp_path, dtype):
    """the same sequence whole, one token at a time and in portions down to two tokens: same logits at every position.  Portions start and end on both sides of the
    temperature's steps, of the attention's 64-key steps and 32-row tiles and of the switch between the few-row and the tiled forms"""
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=3)
    e = engine_for(folder, dtype)
    toks = tokens_for(cfg, 150, seed=4)
    ref, _ = O.forward(cfg, w, toks)
    s = e.seq_acquire()
    whole = e.seq_forward(s, toks)
    e.seq_release(s)
    assert close(cfg, w, toks, whole, ref, dtype)
    s = e.seq_acquire()
    one = np.concatenate([e.seq_forward(s, toks[i:i + 1]) for i in range(len(toks))])
    e.seq_release(s)
    assert close(cfg, w, toks, one, ref, dtype)
    for cuts in ([2, 9, 3, 8, 17, 2, 30, 1, 5, 64, 2, 7], [23, 2, 2, 2, 19, 48, 1, 1, 1, 24, 27], [2] * 75):
        s = e.seq_acquire()
        parts, at = [], 0
        for n in cuts:
            parts.append(e.seq_forward(s, toks[at:at + n]))
            at += n
        assert at == len(toks) and e.seq_length(s) == at
        cut = np.concatenate(parts)
        e.seq_release(s)
        assert close(cfg, w, toks, cut, ref, dtype), cuts
        if dtype == "float32":
            assert rel(one, whole) < 1e-5 and rel(cut, whole) < 1e-5
    e.close()


def test_first_tokens_of_a_sequence(tmp_path):
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=5)
    e = engine_for(folder)
    for n in (1, 2, 3, 4, 5, 6, 8, 9):
        toks = tokens_for(cfg, n, seed=n)
        s = e.seq_acquire()
        assert rel(e.seq_forward(s, toks), O.forward(cfg, w, toks)[0]) < TOL["float32"]
        e.seq_release(s)
    e.close()


def test_slots_side_by_side_used_again_and_cut_back(tmp_path):
    """unequal sequences advance in turn, each alone would give the same; a freed slot (rows of a longer sequence still there) is taken by a shorter one; a slot cut back
    goes on from where it was cut"""
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=6)
    e = engine_for(folder, slots=3)
    all_toks = [tokens_for(cfg, n, k) for k, n in enumerate((60, 33, 7))]
    refs = [O.forward(cfg, w, t)[0] for t in all_toks]
    slots = [e.seq_acquire() for _ in all_toks]
    assert len(set(slots)) == 3
    with pytest.raises(Exception):
        e.seq_acquire()
    cuts = [[20, 1, 1, 30, 8], [2, 1, 25, 5], [1, 1, 5]]
    got, at = [[], [], []], [0, 0, 0]
    for k in range(5):
        for i in range(3):
            if k < len(cuts[i]):
                got[i].append(e.seq_forward(slots[i], all_toks[i][at[i]:at[i] + cuts[i][k]]))
                at[i] += cuts[i][k]
    for i in range(3):
        assert rel(np.concatenate(got[i]), refs[i]) < TOL["float32"], i
    e.seq_release(slots[0])
    c = e.seq_acquire()
    assert c == slots[0]
    tc = tokens_for(cfg, 9, 3)
    assert rel(e.seq_forward(c, tc), O.forward(cfg, w, tc)[0]) < TOL["float32"]
    more = tokens_for(cfg, 30, 5)                                            # its neighbour is untouched
    assert rel(e.seq_forward(slots[1], more), O.forward(cfg, w, all_toks[1] + more)[0][33:]) < TOL["float32"]
    e.seq_truncate(slots[1], 21)
    again = tokens_for(cfg, 14, 8)
    assert rel(e.seq_forward(slots[1], again), O.forward(cfg, w, all_toks[1][:21] + again)[0][21:]) < TOL["float32"]
    e.close()


@pytest.mark.parametrize("how", ["whole", "decoded", "portions"])
def test_distance_and_position_show_in_the_logits(tmp_path, how):
    """a hand-made model: token A's key answers token B's query far above everything else.  The attention layer's first head (steep slope) no longer sees A from far away, its
    last one and the latent layer do; logit 5 / 6 / 7 of a B say what head 0 / head 3 / the latent layer found"""
    W, V, A, B, Z = 24, 8, 1, 2, 3
    cfg = O.config([O.layer_attention(heads=4, kv_heads=1, dim=4, coef=0, scale=1.0), O.layer_latent(heads=1, dim=4, vdim=2, kv_rank=4, scale=1.0)], vocab=V, width=W)
    w = {k: np.zeros(s) for k, s in O.shapes_of(cfg).items()}
    for t in range(V):
        w["embed"][t, t] = 64.0                                              # (far above the position vector's ones)
    for nm in w:
        if "norm" in nm:
            w[nm][:] = 1.0
    p = "l0.mix."
    w[p + "q.norm"][:], w[p + "k.norm"][:] = 4.0, 4.0                        # q.k of a pair (B, A): 4 * 4 * 4
    for h in range(4):
        w[p + "q"][4 * h, B] = 1.0
        w[p + "q"][4 * h + 1, [A, Z]] = 1.0
    w[p + "k"][0, A], w[p + "k"][2, B], w[p + "k"][3, Z] = 1.0, 1.0, 1.0
    w[p + "g"][:, :] = 0.0
    w[p + "o"][16, 0], w[p + "o"][17, 12] = 1.0, 1.0                         # the A entry of the value, of head 0 and of head 3
    w["l0.norm1"][:] = 32.0
    p = "l1.mix."
    w[p + "q"][0, B] = 1.0
    w[p + "dkv"][0, A], w[p + "dkv"][1, B], w[p + "dkv"][2, Z] = 1.0, 1.0, 1.0
    w[p + "uk"][0, 0], w[p + "uv"][0, 0] = 2.0, 1.0
    w[p + "uv"][1, 1:] = 0.01
    w[p + "o"][18, 0], w[p + "o"][19, 1] = 1.0, 1.0
    w["l1.norm1"][:] = 32.0
    w["head"][5, 16], w["head"][6, 17], w["head"][7, 18] = 1.0, 1.0, 1.0
    w = {k: O.to_bf16(v) for k, v in w.items()}
    folder = str(tmp_path / "edge")
    O.save_model(folder, cfg, w)
    e = engine_for(folder)
    n = 200
    for a_at in (0, 31, 32, 63, 64, 100):
        toks = [Z] * n
        toks[a_at] = A
        bs = [p for p in (a_at + 1, a_at + 64, a_at + 65, n - 1) if p < n]
        for b in bs:
            toks[b] = B
        ref, _ = O.forward(cfg, w, toks)
        s = e.seq_acquire()
        if how == "whole":
            got = e.seq_forward(s, toks)
        elif how == "decoded":
            got = np.concatenate([e.seq_forward(s, [t]) for t in toks])
        else:
            got = np.concatenate([e.seq_forward(s, toks[i:i + 13]) for i in range(0, n, 13)])
        e.seq_release(s)
        assert rel(got, ref) < TOL["float32"], a_at
        for b in bs:
            far = b - a_at
            assert (got[b, 6] > 0.3) and (got[b, 7] > 0.3), (a_at, b, got[b, 5:])         # slope 1/256: a lead of dozens outlasts any distance here
            if far <= 1:
                assert got[b, 5] > 0.3
    e.close()


@pytest.mark.parametrize("change", ["slopes", "temperature", "raw values", "head norm", "gate", "latent gate", "shared latents", "correction", "groups", "identity", "shared gate", "position", "post norm"])
def test_every_mechanism_moves_the_logits_of_the_test_model(tmp_path, change, monkeypatch):
    """the oracle with ONE mechanism changed lies far outside the tolerance that the product meets: the comparisons above would notice its absence"""
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=2)
    toks = tokens_for(cfg, 60, seed=3)
    e = engine_for(folder)
    s = e.seq_acquire()
    got = e.seq_forward(s, toks)
    e.close()
    assert rel(got, O.forward(cfg, w, toks)[0]) < TOL["float32"]
    c2, w2 = json.loads(json.dumps(cfg)), dict(w)
    if change == "slopes": monkeypatch.setattr(O, "slope", lambda h, H: 2.0 ** (-8.0 * h / H))
    elif change == "temperature": c2["layers"][1]["mixer"]["q_temp"]["every"] += 1
    elif change == "raw values":
        real = O.attend
        monkeypatch.setattr(O, "attend", lambda q, k, v, pos0, scale, slopes=None: real(q, k, k if slopes is not None else v, pos0, scale, slopes))
    elif change == "head norm":
        real = O.rms
        monkeypatch.setattr(O, "rms", lambda x, w_, eps: x * w_ if x.ndim == 3 else real(x, w_, eps))
    elif change == "gate": w2["l3.mix.g"] = w["l3.mix.g"] * 0.0
    elif change == "latent gate": w2["l4.mix.g"] = w["l4.mix.g"] * 0.0
    elif change == "shared latents": del c2["layers"][2]["mixer"]["kv_from"]; w2["l2.mix.dkv"], w2["l2.mix.dkv.norm"] = w["l0.mix.dkv"], w["l0.mix.dkv.norm"]
    elif change == "correction": w2["l1.mlp.correction"] = w["l1.mlp.correction"] * 0.0
    elif change == "groups": del c2["layers"][1]["mlp"]["router"]["groups"]
    elif change == "identity":
        real = O.plain_unit
        c2["layers"][1]["mlp"]["router"].update(experts=12)
        monkeypatch.setattr(O, "plain_unit", lambda h, w_, pre: 0.0 * h if pre.endswith((".e9.", ".e10.", ".e11.")) else real(h, w_, pre))
    elif change == "shared gate": w2["l1.mlp.shared.sg"] = w["l1.mlp.shared.sg"] * 0.0
    elif change == "position": monkeypatch.setattr(O, "sinusoid", lambda p, width: np.zeros(width))
    else: w2["l2.norm2"] = np.ones_like(w["l2.norm2"])
    assert rel(got, O.forward(c2, w2, toks)[0]) > 10 * TOL["float32"], change


def _other():
    A, L, D, M = O.layer_attention, O.layer_latent, O.dense, O.moe
    return {
        "one of everything": O.config([L(1, 1, 1, 1, mlp=D(1)), A(1, 1, 1, every=1, mlp=M(1, 1, 1)), L(1, 1, 1, 1, kv_from=0, mlp=M(1, 1, 1, identity=1, shared=1))], vocab=5, width=8),
        "all sizes equal, factors one": O.config([L(4, 16, 16, 16, scale=1.0, mlp=D(16)), A(4, 4, 16, coef=1.0, every=1, scale=1.0, mlp=M(4, 4, 16, identity=4, groups=(4, 4), shared=16)),
                                                  L(4, 16, 16, 16, kv_from=0, scale=1.0, mlp=D(16))], vocab=16, width=16),
        "multiples of nothing": O.config([L(3, 7, 5, 11, mlp=M(7, 5, 9, identity=4, shared=13)), A(9, 3, 13, every=5, mlp=D(29)), L(5, 3, 9, 11, kv_from=0, mlp=M(6, 2, 17, identity=3, groups=(3, 1)))], vocab=31, width=23),
        "large heads and latents": O.config([L(2, 136, 200, 264, mlp=D(40)), A(4, 1, 136, mlp=None), L(3, 20, 72, 264, kv_from=0)], vocab=50, width=64),
        "a latent of the largest size": O.config([L(2, 24, 40, 512, mlp=D(24)), L(4, 16, 8, 512, kv_from=0)], width=48),
        "two sources, readers across each other": O.config([L(kv_rank=16), L(kv_rank=24, heads=2), A(mlp=D()), L(kv_from=0, kv_rank=16, heads=8, dim=4), L(kv_from=1, kv_rank=24), L(kv_from=0, kv_rank=16, mlp=M(4, 2, 8))]),
        "attention only, no feed-forward": O.config([A(), A(8, 8, 6, coef=0), A(12, 2, 10, every=3)], eps=1e-2),
        "latent only": O.config([L(mlp=M(3, 3, 12)), L(heads=8, dim=6, vdim=3)]),
        "half of the choices identity": O.config([A(mlp=M(4, 3, 12, identity=4, groups=(2, 1), shared=8)), L(mlp=M(1, 2, 12, identity=5, groups=(3, 2)))]),
        "many experts": O.config([A(mlp=M(130, 9, 8, identity=14, groups=(12, 5), shared=24)), L(mlp=M(250, 20, 8, identity=5))], vocab=40),
        "six heads (slopes between the powers of two)": O.config([A(6, 2, 20, mlp=D()), A(5, 5, 12, mlp=D()), A(16, 1, 4)], eps=1e-6),
        "experts wider than one row of activations": O.config([A(mlp=M(3, 2, 18500, identity=1, shared=40)), L(mlp=M(2, 2, 32))], width=8),
        "wider than one register pass": O.config([L(2, 8, 8, 16, mlp=D(16)), A(2, 1, 8, mlp=M(3, 2, 16, identity=1, shared=8))], vocab=20, width=4104),
    }


OTHER = _other()


@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_sizes(tmp_path, name):
    cfg = OTHER[name]
    folder, w = make(tmp_path, cfg, seed=7)
    toks = tokens_for(cfg, 70, seed=8)
    streams = []
    ref, _ = O.forward(cfg, w, toks, layers_out=streams)
    moe = any((L.get("mlp") or {}).get("kind") == "moe" for L in cfg["layers"])
    for dtype in ("float32", "bfloat16"):
        e = engine_for(folder, dtype)
        e.seq_capture(True)
        s = e.seq_acquire()
        got = e.seq_forward(s, toks[:61])
        cap = e.seq_captured(61)
        e.seq_capture(False)
        tail = np.concatenate([e.seq_forward(s, toks[61:63])] + [e.seq_forward(s, [t]) for t in toks[63:]])
        every = np.concatenate([got, tail])
        e.close()
        if dtype == "float32" or not moe:
            assert rel(cap[-1], streams[-1][:61]) < TOL[dtype] and rel(every, ref) < TOL[dtype], dtype
        else:                                                                # (a close choice of experts may turn: most rows stay close)
            assert np.median(row_err(every, ref)) < TOL[dtype], dtype


def test_long_decoding_and_a_prompt_longer_than_one_internal_pass(tmp_path):
    """1100 tokens are two internal passes: positions, temperature and latents of the second go on from the first; then 200 tokens one by one"""
    cfg = O.config([O.layer_attention(every=100, mlp=O.dense()), O.layer_latent(mlp=O.moe(4, 2, 12, identity=1, shared=12)), O.layer_latent(kv_from=1, heads=2)])
    folder, w = make(tmp_path, cfg, seed=9)
    toks = tokens_for(cfg, 1100, seed=10)
    e = engine_for(folder, ctx=1300)
    s = e.seq_acquire()
    got = e.seq_forward(s, toks, want=[0, 1023, 1024, 1099])
    ref, _ = O.forward(cfg, w, toks)
    assert rel(got, ref[[0, 1023, 1024, 1099]]) < TOL["float32"]
    e.seq_release(s)
    s = e.seq_acquire()
    e.seq_forward(s, toks[:900], want=[])
    dec = np.concatenate([e.seq_forward(s, [t]) for t in toks[900:]])
    assert rel(dec, ref[900:]) < TOL["float32"] and row_err(dec, ref[900:]).max() < 3 * TOL["float32"]
    with pytest.raises(Exception):                                          # the slot's positions are used up
        e.seq_forward(s, toks[:300])
    e.close()


def test_greedy_generation_through_the_engine_and_the_command_line(tmp_path):
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=15, gain=2.0)
    prompt = tokens_for(cfg, 12, seed=16)
    want = O.greedy(cfg, w, prompt, 10)
    e = engine_for(folder)
    assert e.is_sequence_model and e.vocab_size == cfg["vocab"] and e.hidden_size == cfg["width"] and e.n_layers == 5
    assert e.generate_tokens(prompt, 10, temperature=0.0, stop_at_eos=False) == want
    assert e.generate_tokens(prompt, 10, temperature=0.0, stop_at_eos=False) == want      # the slot came back, its old rows are not read
    a = e.generate_tokens(prompt, 8, temperature=0.9, top_k=20, top_p=0.95, seed=5, stop_at_eos=False)
    assert a == e.generate_tokens(prompt, 8, temperature=0.9, top_k=20, top_p=0.95, seed=5, stop_at_eos=False) and len(a) == 8
    assert rel(e.forward(prompt[:8], 0), O.forward(cfg, w, prompt[:8])[0][-1]) < TOL["float32"]
    assert rel(e.forward(prompt[8:], 8), O.forward(cfg, w, prompt)[0][-1]) < TOL["float32"]
    assert rel(e.forward(prompt[3:6], 3), O.forward(cfg, w, prompt[:6])[0][-1]) < TOL["float32"]     # (back to an earlier position)
    e.close()
    cli = os.path.join(ROOT, "ntransformer_amd", "ntransformer")
    r = subprocess.run([cli, "-m", folder, "--dtype", "float32", "--tokens", ",".join(map(str, prompt)), "-n", "10", "-t", "0", "--repeat-penalty", "1"],
                       capture_output=True, text=True, timeout=120)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [int(t) for t in r.stdout.strip().splitlines()[-1].split(",")] == want


def test_trace_runner_replays_steps(tmp_path):
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=17)
    ta, tb = tokens_for(cfg, 40, 1), tokens_for(cfg, 6, 2)
    ra, rb = O.forward(cfg, w, ta)[0], O.forward(cfg, w, tb)[0]
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": ta[:23], "want": [0, 22]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": ta[23:25], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": ta[25:], "want": [14]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "b", "tokens": tb, "want": [5]}], "end": ["b"]},
    ]
    V = cfg["vocab"]
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / ("out_" + dtype)
        out.mkdir()
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out), "--max-tokens", "40"],
                           input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % k for k in range(4)]
        assert not (out / "1.f32").exists()
        got = [np.fromfile(out / ("%d.f32" % k), np.float32).reshape(-1, V) for k in (0, 2, 3)]
        errs = np.concatenate([row_err(a, b) for a, b in zip(got, (ra[[0, 22]], ra[[39]], rb[[5]]))])
        assert (errs.max() if dtype == "float32" else np.median(errs)) < TOL[dtype]


@pytest.mark.parametrize("bad", ["mixer type", "tensor", "kv_heads", "kind", "later layer", "chain", "other rank", "other mixer", "vdim", "down", "groups", "top", "correction", "query rows", "every", "expert"])
def test_refused_folders(tmp_path, bad):
    from ntransformer_amd.engine import Engine
    cfg = mixed()
    w = O.random_weights(cfg, 1)
    mx = [L["mixer"] for L in cfg["layers"]]
    rt = cfg["layers"][1]["mlp"]["router"]
    if bad == "mixer type": cfg["layers"][1]["type"] = "delta"
    elif bad == "tensor": del w["l1.mix.k.norm"]
    elif bad == "kv_heads": mx[1]["kv_heads"] = 3
    elif bad == "kind": cfg["layers"][0]["mlp"]["kind"] = "sparse"
    elif bad == "later layer": mx[2]["kv_from"] = 4
    elif bad == "chain": cfg["layers"].append(O.layer_latent(kv_from=2)); w = O.random_weights(cfg, 1)
    elif bad == "other rank": mx[2]["kv_rank"] = 24
    elif bad == "other mixer": mx[2]["kv_from"] = 1
    elif bad == "vdim": mx[1]["vdim"] = 6
    elif bad == "down": w["l0.mlp.down"] = w["l0.mlp.down"][:, :-1]
    elif bad == "groups": rt["groups"]["count"] = 5
    elif bad == "top": rt["top"] = 7
    elif bad == "correction": w["l1.mlp.correction"] = w["l1.mlp.correction"][:7]
    elif bad == "query rows": w["l0.mix.q"], w["l0.mix.g"] = w["l0.mix.q"][:-1], np.concatenate([w["l0.mix.g"], w["l0.mix.g"][:1]])
    elif bad == "every": mx[1]["q_temp"]["every"] = 0
    else: w["l1.mlp.e3.up"] = w["l1.mlp.e3.up"][:-1]
    folder = str(tmp_path / "bad")
    O.save_model(folder, cfg, w)
    e = Engine()
    with pytest.raises(Exception):
        e.load_folder(folder, max_context=64, dtype="float32")
    e.close()
