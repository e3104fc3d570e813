"""Plain float64 restatement of the Zalazen family (the parallel form of the layer stack with grouped-query window attention and a dense gated feed-forward),
one function per mechanism, for the tests: numpy only, loops over tokens and heads, nothing shared with the product.

Notation.  x [T, W] is the stream, matrices are stored [out, in] and applied as h @ M.T.
  rms(x; w)     = x / sqrt(mean(x^2) + eps) * w
  embedding     x_t = E[s_t] * scale + B[r_t],   r_t = (s_{t-1} * a + s_t * b) mod n,   r_0 = n (the table has n + 1 rows)
  layer         x <- x + attention(rms(x; n1)) + ff(rms(x; n2))          (both of the same x; ff only where the layer has one)
  attention     q, k: the WHOLE projection rms-normed with its weight, then rotated per head (half against half, blended frequencies); position i sees j <= i with
                i - j < size or j < kept; a learned sink per head in the softmax; one gate per head; a layer may read the keys and values of an earlier layer
  feed-forward  D (silu(G h) * (U h))
  logits        head @ rms(x; final)
"""
import json
import math
import os
import struct

import numpy as np

F = np.float64


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


# ---------------------------------------------------------------------------------------------------------------- embedding
def bigram_row(prev, cur, bg):
    """prev None: the sequence's first token"""
    return bg["buckets"] if prev is None else (prev * bg["mul_prev"] + cur * bg["mul_cur"]) % bg["buckets"]


def embed(cfg, w, tokens, prev=None):
    e = cfg["embedding"]
    out = []
    for t in tokens:
        row = w["embed"][t] * e["scale"]
        if e.get("bigram"):
            row = row + w["bigram"][bigram_row(prev, t, e["bigram"])]
        out.append(row)
        prev = t
    return np.array(out, F)


# ---------------------------------------------------------------------------------------------------------------- rotation
def blended_frequencies(rot):
    """(f [dims / 2], magnitude): base^(-2i/dims), and with 'scaling' a blend between f and f / factor along a ramp over the pair index"""
    dims, base = rot["dims"], rot["base"]
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], F)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    def where(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_halves(x, pos, freq, mag, dims):
    """x [..., n]: entry i < dims/2 is paired with entry i + dims/2; the rest passes"""
    half = dims // 2
    a = pos * freq
    c, s = np.cos(a) * mag, np.sin(a) * mag
    y = np.array(x, F)
    u, v = x[..., :half], x[..., half:dims]
    y[..., :half] = u * c - v * s
    y[..., half:dims] = v * c + u * s
    return y


def rotate_rows(z, n_heads, pos0, rot):
    """z [T, n_heads * dn] at positions pos0 .. -> [T, n_heads, dn]"""
    z = z.reshape(z.shape[0], n_heads, -1)
    if not rot:
        return z
    f, mag = blended_frequencies(rot)
    return np.stack([rotate_halves(z[t], pos0 + t, f, mag, rot["dims"]) for t in range(z.shape[0])])


# ---------------------------------------------------------------------------------------------------------------- attention
def sees(i, j, size, kept):
    """query position i, key position j; size None or 0: plain causal"""
    return j <= i and (not size or i - j < size or j < kept)


def sink_softmax(s, sink):
    """exp(s_j) / (exp(sink) + sum exp(s)); sink None: the plain softmax"""
    m = float(np.max(s)) if sink is None else max(float(np.max(s)), sink)
    e = np.exp(s - m)
    return e / (e.sum() + (math.exp(sink - m) if sink is not None else 0.0))


def attend(q, k, v, pos0, scale, size=None, kept=0, sinks=None):
    """q [T, H, dn] at positions pos0 ..; k [P, G, dn], v [P, G, dv] of positions 0 .. P - 1; sinks [H] -> [T, H, dv]"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]), F)
    for t in range(T):
        p = pos0 + t
        js = [j for j in range(p + 1) if sees(p, j, size, kept)]
        kk, vv = k[js], v[js]
        for hh in range(H):
            g = hh // (H // G)
            out[t, hh] = sink_softmax((kk[:, g] @ q[t, hh]) * scale, None if sinks is None else float(sinks[hh])) @ vv[:, g]
    return out


def attention(h, w, pre, mx, eps, pos0=0, past=None, shared=None):
    """h [T, W] at positions pos0 ..; past = (k, v) of this layer's earlier positions; shared = (k, v) of the layer it reads, up to and with these tokens
    -> (out [T, W], (k, v) so far; None where it keeps none of its own)"""
    T = h.shape[0]
    H, G = mx["heads"], mx.get("kv_heads", mx["heads"])
    q = rotate_rows(rms(h @ w[pre + "q"].T, w[pre + "q.norm"], eps), H, pos0, mx.get("rot"))
    if shared is None:
        k = rotate_rows(rms(h @ w[pre + "k"].T, w[pre + "k.norm"], eps), G, pos0, mx.get("rot"))
        v = (h @ w[pre + "v"].T).reshape(T, G, mx["vdim"])
        if past is not None:
            k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
        keep = (k, v)
    else:
        (k, v), keep = shared, None
    mask = mx.get("mask") or {}
    out = attend(q, k, v, pos0, mx["scale"], mask.get("size"), mask.get("keep_first", 0), w[pre + "sink"])
    out = out * sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return out.reshape(T, -1) @ w[pre + "o"].T, keep


# ---------------------------------------------------------------------------------------------------------------- feed-forward
def gated_unit(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


# ---------------------------------------------------------------------------------------------------------------- the model
class Sequence:
    """what a sequence carries from portion to portion: its length, its last token and, per layer, keys and values"""

    def __init__(self, cfg):
        self.n = 0
        self.last = None
        self.per_layer = [None] * len(cfg["layers"])


def forward(cfg, w, tokens, seq=None, layers_out=None):
    """tokens appended to seq (a new sequence if None) -> logits [T, vocab]; layers_out (a list) receives the stream after every layer"""
    seq = seq if seq is not None else Sequence(cfg)
    eps = cfg["norm"]["eps"]
    x = embed(cfg, w, tokens, seq.last)
    for i, L in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, L["mixer"]
        src = mx.get("kv_from")
        y, kv = attention(rms(x, w[p + "norm1"], eps), w, p + "mix.", mx, eps, seq.n, seq.per_layer[i], seq.per_layer[src] if src is not None else None)
        seq.per_layer[i] = kv
        if L.get("mlp"):
            y = y + gated_unit(rms(x, w[p + "norm2"], eps), w, p + "mlp.")
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    seq.n += len(tokens)
    seq.last = tokens[-1]
    return rms(x, w["final.norm"], eps) @ w["head"].T, seq


def greedy(cfg, w, prompt, n):
    """n tokens, each the argmax of the last position's logits"""
    logits, seq = forward(cfg, w, prompt)
    out = []
    for _ in range(n):
        out.append(int(np.argmax(logits[-1])))
        logits, seq = forward(cfg, w, [out[-1]], seq)
    return out


# ---------------------------------------------------------------------------------------------------------------- configurations and folders
YARN = {"factor": 4.0, "original": 16, "fast": 4.0, "slow": 1.0}


def layer(heads=4, kv_heads=2, dim=8, vdim=8, size=16, kept=3, base=10000.0, dims=None, scaling=None, ff=24, kv_from=None, scale=None, rot=True):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if rot:
        mx["rot"] = {"base": base, "dims": dims if dims is not None else dim}
        if scaling:
            mx["rot"]["scaling"] = dict(scaling)
    if size:
        mx["mask"] = {"size": size, "keep_first": kept}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "attention", "mixer": mx, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab=61, width=32, eps=1e-5, embed_scale=2.5, bigram=(41, 7, 3)):
    cfg = {"architecture": "Zalazen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": layers}
    if bigram:
        cfg["embedding"]["bigram"] = {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}
    return cfg


def shapes_of(cfg):
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    if cfg["embedding"].get("bigram"):
        out["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)
    for i, L in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, L["mixer"]
        H, G, dn, dv = mx["heads"], mx.get("kv_heads", mx["heads"]), mx["dim"], mx["vdim"]
        out[p + "norm1"] = (W,)
        out[p + "mix.q"], out[p + "mix.q.norm"], out[p + "mix.sink"] = (H * dn, W), (H * dn,), (H,)
        out[p + "mix.g"], out[p + "mix.o"] = (H, W), (W, H * dv)
        if mx.get("kv_from") is None:
            out[p + "mix.k"], out[p + "mix.k.norm"], out[p + "mix.v"] = (G * dn, W), (G * dn,), (G * dv, W)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            out[p + "norm2"] = (W,)
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ff, W)
            out[p + "mlp.down"] = (W, ff)
    return out


def to_bf16(a):
    """round to the nearest bfloat16 (ties to even), returned as float64"""
    b = np.asarray(a, np.float32).view(np.uint32).astype(np.uint64)
    b = ((b + 0x7FFF + ((b >> 16) & 1)) >> 16) << 16
    return b.astype(np.uint32).view(np.float32).astype(F)


def random_weights(cfg, seed=1, gain=1.0):
    rng = np.random.default_rng(seed)
    w = {}
    for name, shp in shapes_of(cfg).items():
        last = name.split(".")[-1]
        if "norm" in last:
            a = 1.0 + 0.2 * rng.standard_normal(shp)
        elif last == "sink":
            a = rng.uniform(-1.0, 2.0, shp)
        elif name in ("embed", "bigram"):
            a = rng.standard_normal(shp) / math.sqrt(shp[1])
        else:
            a = rng.standard_normal(shp) * gain / math.sqrt(shp[-1])
        w[name] = to_bf16(a)
    return w


def save_model(folder, cfg, w):
    """config.json + model.safetensors (bfloat16)"""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name in sorted(w):
        a = np.asarray(w[name], np.float32)
        raw = (a.view(np.uint32) >> 16).astype(np.uint16).tobytes()
        header[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    hj = json.dumps(header).encode()
    hj += b" " * ((8 - len(hj) % 8) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(hj)))
        f.write(hj)
        for b in blobs:
            f.write(b)


def load_model(folder):
    """(config, weights as float64) of a folder with a bfloat16 / float32 safetensors file"""
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    with open(os.path.join(folder, "model.safetensors"), "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        header = json.loads(f.read(n))
        data = f.read()
    w = {}
    for name, t in header.items():
        if name == "__metadata__":
            continue
        lo, hi = t["data_offsets"]
        if t["dtype"] == "BF16":
            a = (np.frombuffer(data[lo:hi], np.uint16).astype(np.uint32) << 16).view(np.float32)
        elif t["dtype"] == "F32":
            a = np.frombuffer(data[lo:hi], np.float32)
        else:
            continue
        w[name] = a.astype(F).reshape(t["shape"])
    return cfg, w
