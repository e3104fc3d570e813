"""The Zalazen family (the parallel form of the layer stack with grouped-query attention and one dense gated unit per layer: a sliding window beside which a
sequence's first positions stay visible, a learned sink and one gate per head, queries and keys normed over their whole projection, half-split rotation with
blended frequencies, keys and values of an earlier layer, a bigram row in the embedding) against tests/zalazen_oracle.py -- a float64 restatement that shares
nothing with the product.  Every test makes its own small configuration and random bf16-representable weights, writes them as a model folder and runs them
through the C API (the engine's step function, slot cache and kernels); the operator tests call include/ntk_layers.h directly.

Error measure: rms of the difference over rms of the reference.  float32 mode is held to 2e-4 (observed ~1e-6), bfloat16 mode to 4e-2."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import zalazen_oracle as O  # noqa: E402

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
    """windows of three sizes with and without kept positions, layers that read an earlier one with their own masks and head counts, one without feed-forward"""
    L = O.layer
    return O.config([L(size=24, kept=3, scaling=O.YARN), L(size=10, kept=0, heads=6, vdim=12, dims=4), L(size=40, kept=5, heads=2, kv_from=0, scaling=O.YARN),
                     L(size=17, kept=1, heads=2, vdim=12, dims=4, kv_from=1, ff=0), L(size=0, kv_from=0, scaling=O.YARN, ff=40)], **kw)


# ====================================================================================================================== operators
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("V,W,buckets,mp,mc", [(61, 33, 17, 7, 3), (300, 520, 1, 5, 5), (70000, 8, 50021, 104729, 15485863)])
def test_embedding_row_plus_the_row_of_the_token_pair(dtype, V, W, buckets, mp, mc):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(V)
    E, B = O.to_bf16(g.standard_normal((V, W))), O.to_bf16(g.standard_normal((buckets + 1, W)))
    cfg = {"embedding": {"scale": 3.7, "bigram": {"buckets": buckets, "mul_prev": mp, "mul_cur": mc}}}
    w = {"embed": E, "bigram": B}
    toks = [int(t) for t in g.integers(0, V, 9)] + [V - 1, V - 1]
    got = Lr.embed_bigram(E, B, toks, 12345, 0, 3.7, mp, mc, dtype)                       # (at position 0 the given previous token is not used)
    assert rel(got, O.embed(cfg, w, toks)) < 1e-6
    got = Lr.embed_bigram(E, B, toks, V - 1, 5, 3.7, mp, mc, dtype)
    assert rel(got, O.embed(cfg, w, toks, V - 1)) < 1e-6
    assert rel(Lr.embed_bigram(E, B, [3], 4, 1, 3.7, mp, mc, dtype), O.embed(cfg, w, [3], 4)) < 1e-6


@pytest.mark.parametrize("H,G,dn,dv,dims", [(4, 2, 8, 6, 8), (8, 1, 48, 40, 24), (3, 3, 7, 5, 6), (1, 1, 2, 1, 2), (16, 4, 128, 96, 128), (2, 1, 10, 3, 0)])
@pytest.mark.parametrize("T,pos0", [(1, 0), (1, 777), (5, 30), (40, 100)])
def test_norm_over_the_whole_projection_then_rotation(H, G, dn, dv, dims, T, pos0):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(H * 100 + dims + T)
    q, k, v = f32(g.standard_normal((T, H * dn)) * 3), f32(g.standard_normal((T, G * dn)) * 0.2), f32(g.standard_normal((T, G * dv)))
    q[:, :dn] *= 20.0                                                                     # one loud head: a norm per head would level it
    qn, kn = f32(1 + 0.3 * g.standard_normal(H * dn)), f32(1 + 0.3 * g.standard_normal(G * dn))
    rot = {"base": 500.0, "dims": dims, "scaling": {"factor": 3.0, "original": 200, "fast": 8.0, "slow": 1.0}} if dims else None
    freq, mag = O.blended_frequencies(rot) if dims else (None, 1.0)
    eps = 1e-3
    qr = O.rotate_rows(O.rms(q.astype(F64), qn.astype(F64), eps), H, pos0, rot).reshape(T, -1)
    kr = O.rotate_rows(O.rms(k.astype(F64), kn.astype(F64), eps), G, pos0, rot).reshape(T, -1)
    kw = dict(freq=freq, dims=dims, mag=mag, layout=Lr.ROT_HALVES, norm_eps=eps)
    cache, gq, _ = Lr.window_prepare_ex(q, k, v, H, G, dn, dv, pos0, q_norm=qn, k_norm=kn, **kw)
    assert rel(gq, qr) < 1e-5 and rel(cache[pos0:, :G * dn], kr) < 1e-5 and np.array_equal(cache[pos0:, G * dn:], v) and not cache[:pos0].any()
    before = f32(g.standard_normal((pos0 + T, G * (dn + dv))))
    cache, gq, _ = Lr.window_prepare_ex(q, None, None, H, G, dn, dv, pos0, q_norm=qn, cache=before, **kw)         # queries only: the cache is left alone
    assert rel(gq, qr) < 1e-5 and np.array_equal(cache, before)
    qb, kb = f32(g.standard_normal(H * dn)), f32(g.standard_normal(G * dn))               # biases come ahead of the norm
    cache, gq, _ = Lr.window_prepare_ex(q, k, v, H, G, dn, dv, pos0, q_norm=qn, k_norm=kn, qb=qb, kb=kb, **kw)
    assert rel(gq, O.rotate_rows(O.rms(q.astype(F64) + qb, qn.astype(F64), eps), H, pos0, rot).reshape(T, -1)) < 1e-5
    assert rel(cache[pos0:, :G * dn], O.rotate_rows(O.rms(k.astype(F64) + kb, kn.astype(F64), eps), G, pos0, rot).reshape(T, -1)) < 1e-5


def _attention_case(g, H, G, dn, dv, P):
    q = f32(g.standard_normal((P, H * dn)))
    K, V = f32(g.standard_normal((P, G * dn))), f32(g.standard_normal((P, G * dv)))
    return q, K, V, np.concatenate([K, V], axis=1)


def _reference(q, K, V, H, G, dn, dv, pos0, scale, size, kept, sinks):
    T, P = q.shape[0], K.shape[0]
    return O.attend(q.reshape(T, H, dn).astype(F64), K.reshape(P, G, dn).astype(F64), V.reshape(P, G, dv).astype(F64), pos0, scale, size or None, kept, sinks)


@pytest.mark.parametrize("H,G,dn,dv", [(4, 2, 12, 20), (3, 3, 5, 3), (6, 1, 70, 130), (1, 1, 8, 8)])
@pytest.mark.parametrize("pos0,T", [(0, 50), (330, 1), (325, 6), (60, 23)])
@pytest.mark.parametrize("size,kept", [(16, 5), (64, 64), (65, 1), (0, 0), (1, 3), (9, 100), (30, 0)])
def test_attention_over_a_window_beside_kept_first_positions(H, G, dn, dv, pos0, T, size, kept):
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(H * 1000 + pos0 + size)
    P = pos0 + T
    q, K, V, cache = _attention_case(g, H, G, dn, dv, P)
    scale = 1.5 / math.sqrt(dn)
    sinks = f32(g.uniform(-2, 4, H))
    gate = f32(g.standard_normal((T, H)) * 2)
    ref = _reference(q[pos0:], K, V, H, G, dn, dv, pos0, scale, size, kept, sinks)
    for split in (True, False):
        got = Lr.window_attention(q[pos0:], cache, H, G, 1, dn, dv, pos0, size, scale, split=split, keep_first=kept, sinks=sinks)
        assert rel(got, ref.reshape(T, -1)) < 1e-5, split
        got = Lr.window_attention(q[pos0:], cache, H, G, 1, dn, dv, pos0, size, scale, split=split, keep_first=kept, sinks=sinks, gate=gate, head_gate=True)
        assert rel(got, (ref * O.sigmoid(gate.astype(F64))[:, :, None]).reshape(T, -1)) < 1e-5, split
    plain = _reference(q[pos0:], K, V, H, G, dn, dv, pos0, scale, size, kept, None)
    assert rel(Lr.window_attention(q[pos0:], cache, H, G, 1, dn, dv, pos0, size, scale, keep_first=kept), plain.reshape(T, -1)) < 1e-5


def test_a_sink_per_head_takes_its_share_once():
    """all scores zero: n visible keys share 1 / (n + exp(sink)) each, whatever the scale; a high sink leaves all but nothing, a low one all; scores of +-300 stay finite"""
    from ntransformer_amd import layers as Lr
    P, dn, dv = 300, 8, 4
    sinks = f32([-20.0, 0.0, 3.0, 60.0])
    V = f32(np.ones((P, dv)))
    for pos0, T in ((0, P), (P - 1, 1), (200, 7)):
        q, K = np.zeros((T, 4 * dn), np.float32), np.zeros((P, dn), np.float32)
        got = Lr.window_attention(q, np.concatenate([K[:pos0 + T], V[:pos0 + T]], axis=1), 4, 1, 1, dn, dv, pos0, 50, 7.0, keep_first=2, sinks=sinks)
        for t in range(T):
            p = pos0 + t
            n = sum(O.sees(p, j, 50, 2) for j in range(p + 1))
            want = n / (n + np.exp(sinks.astype(F64)))
            assert np.allclose(got[t].reshape(4, dv), want[:, None], rtol=1e-4, atol=1e-12), (pos0, t)
        for s in (-300.0, 300.0):
            q1, K1 = np.full((T, 4 * dn), 1.0, np.float32), np.full((P, dn), s / dn, np.float32)
            got = Lr.window_attention(q1, np.concatenate([K1[:pos0 + T], V[:pos0 + T]], axis=1), 4, 1, 1, dn, dv, pos0, 50, 1.0, keep_first=2, sinks=sinks)
            assert np.isfinite(got).all() and (np.abs(got - (1.0 if s > 0 else 0.0)) < 1e-5).all()


def test_a_towering_key_inside_and_outside_the_window_and_among_the_first():
    """one key's score stands far above the rest: it is returned by exactly the queries that see it -- the last one inside the window, not the next; the last kept
    position for ever, the first one that is not kept no longer than the window -- for a decoded token and inside portions"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(8)
    H, G, dn, dv, size, kept, P = 2, 1, 16, 8, 48, 5, 400
    for tower in (0, 4, 5, 6, 47, 63, 64, 100, 127, 128, 300):
        q, K, V, _ = _attention_case(g, H, G, dn, dv, P)
        q *= 0.05
        d = g.standard_normal(dn)
        d /= np.linalg.norm(d)
        K[tower] = 40.0 * d
        q[:, :dn] += 2.0 * d                                                 # head 0 looks for it everywhere; head 1 does not
        cache = np.concatenate([K, V], axis=1)
        last_in = tower + size - 1
        for pos0, T in ((last_in, 1), (last_in + 1, 1), (last_in - 3, 8), (last_in + 1, 2), (0, min(P, last_in + 30)), (P - 1, 1), (P - 60, 60)):
            if pos0 + T > P or pos0 < 0:
                continue
            got = Lr.window_attention(q[pos0:pos0 + T], cache[:pos0 + T], H, G, 1, dn, dv, pos0, size, 1.0, keep_first=kept, sinks=f32([1.0, -1.0]))
            ref = _reference(q[pos0:pos0 + T], K[:pos0 + T], V[:pos0 + T], H, G, dn, dv, pos0, 1.0, size, kept, [1.0, -1.0]).reshape(T, -1)
            assert rel(got, ref) < 1e-5, (tower, pos0, T)
            for t in range(T):
                p = pos0 + t
                off = np.abs(got[t, :dv] - V[tower]).max()
                if tower <= p <= last_in or (p >= tower and tower < kept):
                    assert off < 1e-3, (tower, p)
                else:
                    assert off > 0.05, (tower, p)


def test_a_far_key_among_hundreds_without_a_mask():
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(9)
    H, G, dn, dv, P = 4, 2, 12, 10, 1300
    for tower in (0, 63, 64, 700, 1279):
        q, K, V, _ = _attention_case(g, H, G, dn, dv, P)
        q *= 0.05
        d = g.standard_normal(dn)
        d /= np.linalg.norm(d)
        K[tower, dn:] = 40.0 * d                                             # key head 1
        q[-1, 2 * dn:3 * dn] += 2.0 * d                                      # query head 2 reads key head 1
        cache = np.concatenate([K, V], axis=1)
        for split in (True, False):
            got = Lr.window_attention(q[-1:], cache, H, G, 1, dn, dv, P - 1, 0, 1.0, split=split, sinks=f32([0.0] * 4))
            assert np.abs(got[0, 2 * dv:3 * dv] - V[tower, dv:]).max() < 1e-3, (tower, split)


def test_gated_unit_into_the_columns_behind_the_heads():
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(4)
    for rows, ff, lda in ((1, 5, 5), (7, 300, 421), (40, 64, 80)):
        gu = f32(g.standard_normal((rows, 2 * ff + 3)) * 2)
        got = Lr.glu_rows(gu, ff, lda)
        assert rel(got[:, :ff], O.silu(gu[:, :ff].astype(F64)) * gu[:, ff:2 * ff]) < 1e-6 and not got[:, ff:].any()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,N,K", [(1, 24, 16), (3, 70, 33), (8, 4200, 264), (1, 5000, 2056), (2, 64, 4104), (1, 40, 9000), (5, 30, 16384)])
def test_few_row_products_with_the_norm_inside_and_onto_the_stream(dtype, T, N, K):
    """the decode products of the family: an RMS norm with a plain weight inside the launch, the gated unit in the epilogue, accumulation"""
    from ntransformer_amd import layers as Lr
    g = np.random.default_rng(N + K)
    x, w, nw, y0 = f32(g.standard_normal((T, K)) * 3), O.to_bf16(g.standard_normal((N, K)) / math.sqrt(K)), f32(1 + 0.3 * g.standard_normal(K)), f32(g.standard_normal((T, N)))
    h = O.rms(x.astype(F64), nw.astype(F64), 1e-3)
    assert rel(Lr.dense(x, w, dtype, norm_w=nw, norm_eps=1e-3), h @ w.T) < 1e-5
    assert rel(Lr.dense(x, w, dtype), x.astype(F64) @ w.T) < 1e-5
    assert rel(Lr.dense(x, w, dtype, y0=y0), y0 + x.astype(F64) @ w.T) < 1e-5
    gu = h @ w.T
    got = Lr.dense(x, w, dtype, norm_w=nw, norm_eps=1e-3, glu_limit=float("inf"), glu_alpha=1.0, glu_up_offset=0.0)
    assert rel(got, O.silu(gu[:, :N // 2]) * gu[:, N // 2:]) < 1e-5


# ====================================================================================================================== whole models
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_with_the_stream_after_every_layer(tmp_path, dtype):
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=2)
    toks = tokens_for(cfg, 60, seed=3)
    streams = []
    ref, _ = O.forward(cfg, w, toks, layers_out=streams)
    e = engine_for(folder, dtype)
    assert e.layer_runs == 5
    e.seq_capture(True)
    s = e.seq_acquire()
    got = e.seq_forward(s, toks)
    cap = e.seq_captured(len(toks))
    for i in range(5):
        assert rel(cap[i], streams[i]) < TOL[dtype], i
    assert rel(got, ref) < TOL[dtype]
    e.seq_capture(False)
    e.seq_release(s)
    s = e.seq_acquire()
    some = e.seq_forward(s, toks, want=[0, 7, 59])                           # wanted places only
    assert rel(some, ref[[0, 7, 59]]) < TOL[dtype]
    e.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prefill_against_token_by_token_and_portions(tmp_path, dtype):
    """the same sequence whole, one token at a time and in portions down to two tokens: same logits at every position.  Portions start and end on both sides of the
    windows' edges, of the kept positions, of the attention's 64-key steps and of the switch between the few-row and the tiled products"""
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=3)
    e = engine_for(folder, dtype)
    toks = tokens_for(cfg, 150, seed=4)
    ref, _ = O.forward(cfg, w, toks)
    s = e.seq_acquire()
    whole = e.seq_forward(s, toks)
    e.seq_release(s)
    assert rel(whole, ref) < TOL[dtype] and row_err(whole, ref).max() < 3 * TOL[dtype]
    s = e.seq_acquire()
    one = np.concatenate([e.seq_forward(s, toks[i:i + 1]) for i in range(len(toks))])
    e.seq_release(s)
    assert rel(one, ref) < TOL[dtype] and row_err(one, ref).max() < 3 * TOL[dtype]
    for cuts in ([2, 9, 3, 8, 17, 2, 30, 1, 5, 64, 2, 7], [23, 2, 2, 2, 19, 48, 1, 1, 1, 24, 27], [2] * 75):
        s = e.seq_acquire()
        parts, at = [], 0
        for n in cuts:
            parts.append(e.seq_forward(s, toks[at:at + n]))
            at += n
        assert at == len(toks) and e.seq_length(s) == at
        cut = np.concatenate(parts)
        e.seq_release(s)
        assert rel(cut, ref) < TOL[dtype] and row_err(cut, ref).max() < 3 * TOL[dtype], cuts
        if dtype == "float32":
            assert rel(one, whole) < 1e-5 and rel(cut, whole) < 1e-5
    e.close()


def test_first_tokens_of_a_sequence(tmp_path):
    cfg = mixed()
    folder, w = make(tmp_path, cfg, seed=5)
    e = engine_for(folder)
    for n in (1, 2, 3, 4, 5, 6):
        toks = tokens_for(cfg, n, seed=n)
        s = e.seq_acquire()
        assert rel(e.seq_forward(s, toks), O.forward(cfg, w, toks)[0]) < TOL["float32"]
        e.seq_release(s)
    e.close()


def test_the_bigram_row_follows_the_cut(tmp_path):
    """a table whose rows are far larger than the embedding's: a portion's first token takes the row of the token before it, a sequence's first token the last row,
    also in a slot that another sequence held before and after the slot was cut back"""
    cfg = mixed(embed_scale=0.5)
    folder, w = make(tmp_path, cfg, seed=21, change=lambda w: w.update(bigram=O.to_bf16(w["bigram"] * 8.0)))
    e = engine_for(folder)
    toks = tokens_for(cfg, 40, seed=22)
    ref, _ = O.forward(cfg, w, toks)
    s = e.seq_acquire()
    got = [e.seq_forward(s, toks[:1]), e.seq_forward(s, toks[1:3]), e.seq_forward(s, toks[3:30]), e.seq_forward(s, toks[30:])]
    assert rel(np.concatenate(got), ref) < TOL["float32"]
    e.seq_truncate(s, 17)                                                    # cut back: the token at place 16 is the one before
    again = toks[17:20] + [toks[0]] * 3
    assert rel(e.seq_forward(s, again), O.forward(cfg, w, toks[:17] + again)[0][17:]) < TOL["float32"]
    e.seq_truncate(s, 1)
    assert rel(e.seq_forward(s, toks[5:9]), O.forward(cfg, w, toks[:1] + toks[5:9])[0][1:]) < TOL["float32"]
    e.seq_release(s)
    s = e.seq_acquire()
    assert rel(e.seq_forward(s, toks[7:19]), O.forward(cfg, w, toks[7:19])[0]) < TOL["float32"]
    e.close()


def test_slots_side_by_side_and_a_slot_used_again(tmp_path):
    """unequal sequences advance in turn, each alone would give the same; a freed slot (rows and tokens of a longer sequence still there) is taken by a shorter one"""
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
    e.close()


@pytest.mark.parametrize("how", ["whole", "decoded", "portions"])
def test_edges_of_window_and_kept_positions_show_in_the_logits(tmp_path, how):
    """one attention layer whose queries and keys are driven by the token: token A's key answers token B's query alone and far above the sink, so a B sees whether an
    A lies inside its window or among the kept first positions; every other place is filled with a token whose key stays low"""
    W, V, A, B, Z = 16, 8, 1, 2, 3
    size, kept = 20, 4
    cfg = O.config([O.layer(heads=2, kv_heads=1, dim=4, vdim=4, size=size, kept=kept, ff=0, scale=1.0, rot=False)], vocab=V, width=W, embed_scale=1.0, bigram=None)
    w = {k: np.zeros(s) for k, s in O.shapes_of(cfg).items()}
    for t in range(V):
        w["embed"][t, t] = 1.0
    for nm in ("l0.norm1", "l0.mix.q.norm", "l0.mix.k.norm", "final.norm"):
        w[nm][:] = 1.0
    w["l0.mix.q.norm"][:] = 4.0
    w["l0.mix.q"][0, B] = w["l0.mix.k"][0, A] = 1.0                          # score of (B, A): (2 sqrt 2 x 4) x 2, of anything else 0
    w["l0.mix.q"][1, :] = w["l0.mix.k"][2, :] = 0.1
    w["l0.mix.k"][2, A] = 0.0
    w["l0.mix.v"][0, A] = 1.0
    w["l0.mix.sink"][:] = 4.0
    w["l0.mix.g"][:, :] = 1.0
    w["l0.mix.o"][8, 0] = 2.0
    w["head"][5, 8] = 1.0
    w = {k: O.to_bf16(v) for k, v in w.items()}
    folder = str(tmp_path / "edge")
    O.save_model(folder, cfg, w)
    e = engine_for(folder)
    seen = {}
    n = 90
    for a_at in (0, kept - 1, kept, kept + 1, 30):
        toks = [Z] * n
        toks[a_at] = A
        bs = [p for p in (a_at + 1, a_at + size - 1, a_at + size, a_at + size + 1, n - 1) if p < n]
        for p in bs:
            toks[p] = B
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
        for p in bs:
            inside = p - a_at < size or a_at < kept
            assert (got[p, 5] > 1.0) == inside, (a_at, p, got[p, 5])
            seen[inside] = seen.get(inside, 0) + 1
    assert seen[True] >= 10 and seen[False] >= 5
    e.close()


@pytest.mark.parametrize("change", ["sink", "gate", "kept", "window", "mag", "norm", "shared"])
def test_every_mechanism_moves_the_logits_of_the_test_model(tmp_path, change):
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
    if change == "sink": w2["l0.mix.sink"] = w["l0.mix.sink"] - 30.0
    elif change == "gate": w2["l1.mix.g"] = w["l1.mix.g"] * 0.0
    elif change == "kept": c2["layers"][0]["mixer"]["mask"]["keep_first"] -= 1
    elif change == "window": c2["layers"][1]["mixer"]["mask"]["size"] += 1
    elif change == "mag": c2["layers"][0]["mixer"]["rot"]["scaling"]["factor"] = 1.0
    elif change == "norm": w2["l0.mix.k.norm"] = np.ones_like(w["l0.mix.k.norm"])
    else: c2["layers"][4]["mixer"]["kv_from"] = 1; c2["layers"][4]["mixer"]["vdim"] = 12; w2["l4.mix.o"] = np.concatenate([w["l4.mix.o"], w["l4.mix.o"][:, :16]], axis=1)
    assert rel(got, O.forward(c2, w2, toks)[0]) > 10 * TOL["float32"], change


def _other():
    L = O.layer
    return {
        "one of everything": O.config([L(heads=1, kv_heads=1, dim=2, vdim=1, size=1, kept=1, ff=1), L(heads=1, kv_heads=1, dim=2, vdim=1, size=2, kept=0, ff=1, kv_from=0)],
                                      vocab=5, width=8, bigram=(1, 1, 1)),
        "all sizes equal, factors one": O.config([L(heads=4, kv_heads=4, dim=16, vdim=16, size=16, kept=16, ff=16, scale=1.0, scaling={"factor": 1.0, "original": 16, "fast": 1.0, "slow": 1.0}),
                                                  L(heads=4, kv_heads=4, dim=16, vdim=16, size=16, kept=16, ff=16, scale=1.0)], vocab=16, width=16, embed_scale=1.0, bigram=(16, 1, 1)),
        "multiples of nothing": O.config([L(heads=3, kv_heads=1, dim=7, vdim=5, dims=6, size=19, kept=2, ff=29), L(heads=6, kv_heads=3, dim=9, vdim=5, dims=2, size=7, kept=9, ff=17),
                                          L(heads=9, kv_heads=3, dim=9, vdim=5, dims=2, size=11, kept=1, ff=0, kv_from=1)], vocab=31, width=23),
        "wide heads": O.config([L(heads=2, kv_heads=1, dim=136, vdim=200, dims=64, size=40, kept=4, ff=40, scaling={"factor": 8.0, "original": 64, "fast": 8.0, "slow": 0.5})], vocab=50, width=64),
        "no mask, no rotation, no bigram": O.config([L(size=0, rot=False), L(size=0, rot=False, kv_from=0)], bigram=None),
        "windows and shared layers in another order": O.config([L(size=0), L(size=5, kept=1, ff=0), L(size=50, kept=2, kv_from=0), L(size=3, kept=0), L(size=33, kept=8, kv_from=3),
                                                                L(size=12, kept=3, kv_from=0, heads=8)]),
        "more kept positions than tokens": O.config([L(size=4, kept=500), L(size=2, kept=60)]),
        "a fully rotated head and a long ramp": O.config([L(dim=24, dims=24, base=1e6, scaling={"factor": 32.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
                                                          L(dim=24, dims=12, base=50.0, scaling={"factor": 2.0, "original": 8, "fast": 100.0, "slow": 0.01})], eps=1e-2),
        "output products apart": O.config([L(ff=16384, size=12), L(ff=16384 - 32, size=9)], width=8),
    }


OTHER = _other()


@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_sizes(tmp_path, name):
    cfg = OTHER[name]
    folder, w = make(tmp_path, cfg, seed=7)
    toks = tokens_for(cfg, 70, seed=8)
    streams = []
    ref, _ = O.forward(cfg, w, toks, layers_out=streams)
    for dtype in ("float32", "bfloat16"):
        e = engine_for(folder, dtype)
        e.seq_capture(True)
        s = e.seq_acquire()
        got = e.seq_forward(s, toks[:61])
        assert rel(e.seq_captured(61)[-1], streams[-1][:61]) < TOL[dtype], dtype
        e.seq_capture(False)
        tail = np.concatenate([e.seq_forward(s, toks[61:63])] + [e.seq_forward(s, [t]) for t in toks[63:]])
        assert rel(got, ref[:61]) < TOL[dtype], dtype
        assert rel(np.concatenate([got, tail]), ref) < TOL[dtype], dtype
        e.close()


def test_long_decoding_and_a_prompt_longer_than_one_internal_pass(tmp_path):
    """1100 tokens are two internal passes: the token before the second pass, the shared rows and the kept positions come from the first; then 200 tokens one by one
    far behind the kept positions, several windows long"""
    cfg = O.config([O.layer(size=88, kept=4), O.layer(size=200, kept=1), O.layer(size=30, kept=7, kv_from=0), O.layer(size=0, kv_from=1, ff=0)])
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
        assert rel(np.fromfile(out / "0.f32", np.float32).reshape(-1, V), ra[[0, 22]]) < TOL[dtype]
        assert rel(np.fromfile(out / "2.f32", np.float32).reshape(-1, V), ra[[39]]) < TOL[dtype]
        assert rel(np.fromfile(out / "3.f32", np.float32).reshape(-1, V), rb[[5]]) < TOL[dtype]


@pytest.mark.parametrize("bad", ["mixer type", "tensor", "kv_heads", "kind", "later layer", "chain", "other sizes", "buckets", "down", "kept"])
def test_refused_folders(tmp_path, bad):
    from ntransformer_amd.engine import Engine
    cfg = mixed()
    w = O.random_weights(cfg, 1)
    mx = [L["mixer"] for L in cfg["layers"]]
    if bad == "mixer type": cfg["layers"][1]["type"] = "delta"
    elif bad == "tensor": del w["l1.mix.sink"]
    elif bad == "kv_heads": mx[1]["kv_heads"] = 4
    elif bad == "kind": cfg["layers"][0]["mlp"]["kind"] = "moe"
    elif bad == "later layer": mx[2]["kv_from"] = 3
    elif bad == "chain": mx[4]["kv_from"] = 2
    elif bad == "other sizes": mx[4]["kv_from"] = 1
    elif bad == "buckets": cfg["embedding"]["bigram"]["buckets"] += 1
    elif bad == "down": w["l0.mlp.down"] = w["l0.mlp.down"][:, :-1]
    else: mx[0]["mask"]["keep_first"] = -1
    folder = str(tmp_path / "bad")
    O.save_model(folder, cfg, w)
    e = Engine()
    with pytest.raises(Exception):
        e.load_folder(folder, max_context=64, dtype="float32")
    e.close()
