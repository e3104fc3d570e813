"""Host side of the Gibevik family (no GPU): the folder reader and the registry know the family, and the float64 restatement's own invariants -- the things the GPU
tests lean on: causality, what is carried across a cut (keys with their raw values, latents), the distance bias, the query temperature, the norm per head, the router
with its correction, groups and identity experts, the shared latents, the position vector, the synthetic folders of the benchmark."""
import ctypes as C
import json
import math
import os
import sys

import numpy as np

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import gibevik_oracle as O  # noqa: E402
from ntransformer_amd import _lib  # noqa: E402


def describe(path):
    L = _lib.lib()
    L.nt_model_folder_describe.argtypes = [C.c_char_p, C.c_char_p, C.c_int]
    n = L.nt_model_folder_describe(path.encode(), None, 0)
    assert n >= 0
    buf = C.create_string_buffer(n + 1)
    assert L.nt_model_folder_describe(path.encode(), buf, n + 1) == n
    return json.loads(buf.value.decode())


def small():
    return O.config([O.layer_latent(mlp=O.dense()), O.layer_latent(kv_from=0, heads=2, vdim=6, mlp=O.moe(7, 3, 10, identity=2, groups=(3, 2), shared=9)),
                     O.layer_attention(mlp=O.moe(4, 1)), O.layer_attention(coef=0, heads=6, kv_heads=3)])


def test_a_written_folder_is_described_and_its_family_is_built_in(tmp_path):
    cfg = small()
    w = O.random_weights(cfg, 3)
    O.save_model(str(tmp_path / "m"), cfg, w)
    d = describe(str(tmp_path / "m"))
    assert d["architecture"] == "Gibevik" and d["family_built_in"] is True and {"Gibevik", "Zalazen", "Fifotar", "Tubazen", "Nizorax", "Fabolorn"} <= set(d["families"])
    got = {t["name"]: tuple(t["shape"]) for t in d["tensors"]}
    assert got == {k: tuple(np.shape(v)) for k, v in w.items()}
    assert "l1.mix.dkv" not in got and "l2.mix.v" not in got and "l3.norm2" not in got and got["l1.mlp.router"] == (9, 32) and "l1.mlp.e7.up" not in got
    c2, w2 = O.load_model(str(tmp_path / "m"))
    assert c2 == cfg and all(np.array_equal(w[k], w2[k]) for k in w)


def test_causality_and_cuts_of_the_whole_model():
    cfg = small()
    w = O.random_weights(cfg, 2)
    toks = [int(t) for t in np.random.default_rng(0).integers(0, cfg["vocab"], 17)]
    streams = []
    lg, _ = O.forward(cfg, w, toks, layers_out=streams)
    assert len(streams) == 4 and streams[0].shape == (17, cfg["width"]) and lg.shape == (17, cfg["vocab"])
    assert np.allclose(lg[:9], O.forward(cfg, w, toks[:9])[0], atol=1e-10)
    seq, parts = None, []
    for a, b in ((0, 5), (5, 6), (6, 8), (8, 17)):
        o, seq = O.forward(cfg, w, toks[a:b], seq)
        parts.append(o)
    assert np.allclose(np.concatenate(parts), lg, atol=1e-9) and seq.n == 17


def test_position_vector():
    u = O.sinusoid(3, 6)
    assert np.allclose(u[:2], [math.sin(3), math.cos(3)]) and np.allclose(u[4:], [math.sin(3 * 10000 ** (-4 / 6)), math.cos(3 * 10000 ** (-4 / 6))])
    assert np.array_equal(O.sinusoid(0, 5), [0, 1, 0, 1, 0])
    w = {"embed": np.arange(12.0).reshape(3, 4)}
    assert np.allclose(O.embed(w, [2, 0], 7), [w["embed"][2] + O.sinusoid(7, 4), w["embed"][0] + O.sinusoid(8, 4)])


def test_distance_bias_temperature_and_heads():
    assert [O.slope(h, 4) for h in range(4)] == [2 ** -2.0, 2 ** -4.0, 2 ** -6.0, 2 ** -8.0] and O.slope(0, 1) == 2 ** -8.0
    qt = {"coef": 0.5, "every": 4}
    assert O.temperature(2, qt) == 1.0 and abs(O.temperature(3, qt) - (1 + 0.5 * math.log(2))) < 1e-15 and O.temperature(3, None) == 1.0
    q, k = np.zeros((1, 2, 3)), np.zeros((5, 1, 3))
    v = np.eye(5)[:, None, :]
    got = O.attend(q, k, v, 4, 1.0, [math.log(2.0), 0.0])                               # equal scores: weights halve with every step back in head 0, are equal in head 1
    assert np.allclose(got[0, 0], np.array([1, 2, 4, 8, 16]) / 31) and np.allclose(got[0, 1], 0.2)


def test_values_are_the_keys_ahead_of_their_norm():
    cfg = O.config([O.layer_attention(heads=1, kv_heads=1, dim=4, coef=0)], width=4)
    w = O.random_weights(cfg, 1)
    w["l0.mix.g"] = np.full((4, 4), 0.0)
    w["l0.mix.o"] = 2.0 * np.eye(4)
    x = np.array([[1.0, 2.0, 3.0, -1.0]])
    y, (k, v) = O.attention(x, w, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)            # one token: it sees itself alone, gate 1/2 times 2
    assert np.allclose(y, x @ w["l0.mix.k"].T) and np.allclose(v[:, 0], y) and np.allclose(k[:, 0], O.rms(v[:, 0], w["l0.mix.k.norm"], 1e-5))


def test_router_correction_groups_and_identity():
    z = np.log(np.array([0.1, 0.2, 0.3, 0.4]))
    assert [e for e, _ in O.route(z, np.zeros(4), 2)] == [3, 2]
    got = O.route(z, np.array([0.0, 0.9, 0.0, -5.0]), 2)
    assert [e for e, _ in got] == [1, 2] and np.allclose([s for _, s in got], [0.2, 0.3])           # chosen with the correction, weighted without it
    assert [e for e, _ in O.route(z, np.array([-3.0, -3.0, -2.0, -9.0]), 2, {"count": 2, "keep": 1})] == [2, 3]      # the best group's second, negative as it is
    cfg = O.config([O.layer_latent(mlp=O.moe(2, 2, 4, identity=1))], width=8)
    w = O.random_weights(cfg, 1)
    w["l0.mlp.correction"] = np.array([-9.0, -9.0, 9.0])
    h = np.arange(8.0)[None] / 8
    s = O.softmax((h @ w["l0.mlp.router"].T)[0])
    other = int(np.argmax(s[:2]))
    assert np.allclose(O.experts(h, w, "l0.mlp.", cfg["layers"][0]["mlp"]), s[2] * h + s[other] * O.plain_unit(h, w, "l0.mlp.e%d." % other))
    assert np.array_equal(O.squared_relu(np.array([-3.0, 0.0, 2.0])), [0.0, 0.0, 4.0])


def test_a_layer_without_latents_of_its_own_reads_the_named_one():
    """giving the reading layer the source's projection of ITS input changes the result: the latents come from the source's input"""
    cfg = small()
    w = O.random_weights(cfg, 4)
    toks = [1, 2, 3, 4, 5, 6]
    ref, _ = O.forward(cfg, w, toks)
    own = json.loads(json.dumps(cfg))
    del own["layers"][1]["mixer"]["kv_from"]
    w2 = dict(w)
    for nm in ("dkv", "dkv.norm"):
        w2["l1.mix." + nm] = w["l0.mix." + nm]
    assert np.abs(O.forward(own, w2, toks)[0] - ref).max() > 1e-2


def test_synthetic_folders_of_the_benchmark_have_the_family_s_tensors(tmp_path):
    from ntransformer_amd import synth_folder as S
    cfg = S.gibevik_config("tiny", layers=4)
    S.write_folder(str(tmp_path / "s"), cfg)
    d = describe(str(tmp_path / "s"))
    assert d["architecture"] == "Gibevik" and d["family_built_in"] is True
    got = {t["name"]: tuple(t["shape"]) for t in d["tensors"]}
    assert got == S.gibevik_shapes(cfg) and got == {k: tuple(v) for k, v in O.shapes_of(cfg).items()}
    assert "l1.mix.dkv" not in got and cfg["layers"][1]["mixer"]["kv_from"] == 0 and "l2.mix.k" in got and "l1.mlp.shared.sg" in got
    big = S.gibevik_config("lite", layers=2)
    rt = big["layers"][1]["mlp"]["router"]
    assert rt["experts"] + rt["identity"] == S.PRESETS["lite"]["experts"] and rt["groups"] == {"count": 4, "keep": 2}
    shared = [k["type"] for k in S.fifotar_config("tiny", 8)["layers"]]
    assert shared == ["attention", "delta", "latent_attention", "delta"] * 2               # (the older benchmark's order is what it was)
