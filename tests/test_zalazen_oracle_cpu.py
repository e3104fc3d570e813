"""Host side of the Zalazen family (no GPU): the folder reader and the registry know the family, and the float64 restatement's own invariants -- the things the
GPU tests lean on: causality, what is carried across a cut (keys and values, the last token), the window with its kept first positions, the sink, the norm over
the whole projection, the blended frequencies, the shared keys and values, the synthetic folders of the benchmark."""
import ctypes as C
import json
import math
import os
import sys

import numpy as np

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import zalazen_oracle as O  # noqa: E402
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
    return O.config([O.layer(size=6, kept=2, scaling=O.YARN), O.layer(size=4, kept=1), O.layer(size=9, kept=3, kv_from=1), O.layer(kv_from=0, size=0, scaling=O.YARN, ff=0)])


def test_a_written_folder_is_described_and_its_family_is_built_in(tmp_path):
    cfg = small()
    w = O.random_weights(cfg, 3)
    O.save_model(str(tmp_path / "m"), cfg, w)
    d = describe(str(tmp_path / "m"))
    assert d["architecture"] == "Zalazen" and d["family_built_in"] is True and {"Zalazen", "Fifotar", "Tubazen", "Nizorax", "Fabolorn"} <= set(d["families"])
    got = {t["name"]: tuple(t["shape"]) for t in d["tensors"]}
    assert got == {k: tuple(np.shape(v)) for k, v in w.items()}
    assert got["bigram"] == (42, 32) and "l2.mix.k" not in got and "l2.mix.k.norm" not in got and "l3.norm2" not in got and got["l1.mix.k.norm"] == (16,)
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
    assert np.allclose(np.concatenate(parts), lg, atol=1e-9) and seq.n == 17 and seq.last == toks[-1]


def test_the_window_and_its_kept_first_positions():
    assert [j for j in range(12) if O.sees(10, j, 4, 2)] == [0, 1, 7, 8, 9, 10]
    assert [j for j in range(12) if O.sees(1, j, 4, 3)] == [0, 1]                       # a kept position still is not seen before its time
    assert [j for j in range(12) if O.sees(5, j, 1, 0)] == [5] and [j for j in range(6) if O.sees(3, j, None, 0)] == [0, 1, 2, 3]


def test_sink_norm_and_bigram_row():
    s = np.array([0.0, math.log(2.0)])
    assert np.allclose(O.sink_softmax(s, math.log(3.0)), [1 / 6, 2 / 6]) and np.allclose(O.sink_softmax(s, None), [1 / 3, 2 / 3])
    assert O.sink_softmax(np.array([-800.0]), 800.0)[0] == 0.0 and abs(O.sink_softmax(np.array([800.0]), -800.0)[0] - 1.0) < 1e-12
    z = np.array([[3.0, 4.0, 0.0, 0.0]])                                                # one norm over all four entries, not over two heads of two
    assert np.allclose(O.rms(z, np.ones(4), 0.0), z / 2.5)
    bg = {"buckets": 11, "mul_prev": 5, "mul_cur": 3}
    assert O.bigram_row(None, 4, bg) == 11 and O.bigram_row(2, 4, bg) == 0 and O.bigram_row(4, 2, bg) == 4


def test_blended_frequencies_and_the_half_split_pairs():
    f, mag = O.blended_frequencies({"base": 100.0, "dims": 8})
    assert np.allclose(f, [1.0, 100 ** -0.25, 0.1, 100 ** -0.75]) and mag == 1.0
    f2, mag2 = O.blended_frequencies({"base": 100.0, "dims": 8, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}})
    assert abs(mag2 - (0.1 * math.log(4.0) + 1.0)) < 1e-15 and f2[0] == f[0] and abs(f2[3] - f[3] / 4.0) < 1e-15 and f[1] / 4 < f2[1] < f[1]
    x = np.arange(1.0, 11.0)
    y = O.rotate_halves(x, 3, f, 1.0, 8)
    a = 3 * f[1]
    assert np.allclose([y[1], y[5]], [x[1] * math.cos(a) - x[5] * math.sin(a), x[5] * math.cos(a) + x[1] * math.sin(a)]) and np.array_equal(y[8:], x[8:])


def test_a_layer_without_keys_of_its_own_reads_the_named_one():
    """giving the reading layer a copy of the source's projections of ITS input changes the result: the keys come from the source's input"""
    cfg = small()
    w = O.random_weights(cfg, 4)
    toks = [1, 2, 3, 4, 5, 6]
    ref, _ = O.forward(cfg, w, toks)
    own = json.loads(json.dumps(cfg))
    del own["layers"][2]["mixer"]["kv_from"]
    w2 = dict(w)
    for nm in ("k", "k.norm", "v"):
        w2["l2.mix." + nm] = w["l1.mix." + nm]
    assert np.abs(O.forward(own, w2, toks)[0] - ref).max() > 1e-2
    other = json.loads(json.dumps(cfg))
    other["layers"][2]["mixer"]["kv_from"] = 0
    assert np.abs(O.forward(other, w, toks)[0] - ref).max() > 1e-2


def test_synthetic_folders_of_the_benchmark_have_the_family_s_tensors(tmp_path):
    from ntransformer_amd import synth_folder as S
    cfg = S.zalazen_config("tiny", layers=4)
    S.write_folder(str(tmp_path / "s"), cfg)
    d = describe(str(tmp_path / "s"))
    assert d["architecture"] == "Zalazen" and d["family_built_in"] is True
    got = {t["name"]: tuple(t["shape"]) for t in d["tensors"]}
    assert got == S.shapes_of(cfg) and got == {k: tuple(v) for k, v in O.shapes_of(cfg).items()}
    assert "l1.mix.k" not in got and "l2.mix.k" in got and cfg["layers"][3]["mixer"]["kv_from"] == 2
