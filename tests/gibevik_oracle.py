"""Plain float64 restatement of the Gibevik family (the post-norm form of the layer stack: grouped-query attention whose values are its raw keys and latent
attention without positions, one gated dense feed-forward or a mixture of squared-relu experts with identity experts), one function per mechanism, for the
tests: numpy only, loops over tokens and heads, nothing shared with the product.

Notation.  x [T, W] is the stream, matrices are stored [out, in] and applied as h @ M.T.
  rms(x; w)     = x / sqrt(mean(x^2) + eps) * w
  embedding     x_p = E[s_p] + u(p),   u(p)_{2i} = sin(p 10000^(-2i/W)),  u(p)_{2i+1} = cos(p 10000^(-2i/W))
  layer         x <- x + rms(mixer(x); n1),   x <- x + rms(ff(x); n2)          (the sublayers read the stream as it is)
  attention     k~ = W_k x, v = k~, k = rms(k~) per head, q = rms(W_q x) per head times 1 + c ln(floor((p + 1) / every) + 1); scores scale q.k - 2^(-8(h+1)/H) (i - j);
                the joined heads times sigmoid(W_g x), element by element
  latent        c = rms(W_dkv x) (or an earlier layer's c), k = W_uk c, v = W_uv c, scores scale q.k; one gate per head
  feed-forward  dense: D (silu(G x) * (U x));  experts: sum over the chosen e of s_e D_e relu(U_e x)^2, identity experts give x; + sigmoid(w . x) shared(x)
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


def squared_relu(z):
    return np.maximum(z, 0.0) ** 2


def rms(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def softmax(z):
    e = np.exp(z - np.max(z))
    return e / e.sum()


# ---------------------------------------------------------------------------------------------------------------- embedding
def sinusoid(p, width):
    out = np.zeros(width, F)
    for n in range(width):
        a = p * 10000.0 ** (-2.0 * (n // 2) / width)
        out[n] = math.cos(a) if n % 2 else math.sin(a)
    return out


def embed(w, tokens, pos0):
    E = w["embed"]
    return np.array([E[t] + sinusoid(pos0 + i, E.shape[1]) for i, t in enumerate(tokens)], F)


# ---------------------------------------------------------------------------------------------------------------- attention
def slope(h, H):
    return 2.0 ** (-8.0 * (h + 1) / H)


def temperature(p, qt):
    """factor on the query at position p; qt None: none"""
    return 1.0 if not qt else 1.0 + qt["coef"] * math.log(math.floor((p + 1) / qt["every"]) + 1)


def attend(q, k, v, pos0, scale, slopes=None):
    """q [T, H, dn] at positions pos0 ..; k [P, G, dn], v [P, G, dv] of positions 0 .. P - 1; slopes [H] or None -> [T, H, dv]"""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]), F)
    for t in range(T):
        p = pos0 + t
        back = p - np.arange(p + 1)
        for hh in range(H):
            g = hh // (H // G)
            s = (k[:p + 1, g] @ q[t, hh]) * scale
            if slopes is not None:
                s = s - slopes[hh] * back
            out[t, hh] = softmax(s) @ v[:p + 1, g]
    return out


def attention(h, w, pre, mx, eps, pos0=0, past=None):
    """h [T, W] at positions pos0 ..; past = (k, v) of the earlier positions -> (out [T, W], (k, v) so far)"""
    T = h.shape[0]
    H, G, dn = mx["heads"], mx.get("kv_heads", mx["heads"]), mx["dim"]
    raw = (h @ w[pre + "k"].T).reshape(T, G, dn)
    k, v = rms(raw, w[pre + "k.norm"], eps), raw
    q = rms((h @ w[pre + "q"].T).reshape(T, H, dn), w[pre + "q.norm"], eps)
    q = q * np.array([temperature(pos0 + t, mx.get("q_temp")) for t in range(T)])[:, None, None]
    if past is not None:
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    out = attend(q, k, v, pos0, mx["scale"], [slope(i, H) for i in range(H)]).reshape(T, -1)
    return (out * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T, (k, v)


def latent_attention(h, w, pre, mx, eps, pos0=0, past=None, shared=None):
    """past = this layer's latents of the earlier positions; shared = the latents of the layer it reads, up to and with these tokens
    -> (out [T, W], latents so far; None where it keeps none of its own)"""
    T = h.shape[0]
    H, dn, dv = mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, dn)
    if shared is None:
        c = rms(h @ w[pre + "dkv"].T, w[pre + "dkv.norm"], eps)
        if past is not None:
            c = np.concatenate([past, c])
        keep = c
    else:
        c, keep = shared, None
    k = (c @ w[pre + "uk"].T).reshape(-1, H, dn)
    v = (c @ w[pre + "uv"].T).reshape(-1, H, dv)
    out = attend(q, k, v, pos0, mx["scale"])
    out = out * sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return out.reshape(T, -1) @ w[pre + "o"].T, keep


# ---------------------------------------------------------------------------------------------------------------- feed-forward
def gated_unit(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def plain_unit(h, w, pre):
    return squared_relu(h @ w[pre + "up"].T) @ w[pre + "down"].T


def route(z, correction, top, groups=None):
    """router outputs of one token -> [(expert, weight)]: chosen by softmax + correction among the best groups, weighted by the softmax alone"""
    s = softmax(z)
    choice = s + correction
    n = len(z)
    if groups:
        per = n // groups["count"]
        best = [max(choice[g * per:(g + 1) * per]) for g in range(groups["count"])]
        kept = sorted(range(groups["count"]), key=lambda g: (-best[g], g))[:groups["keep"]]
        choice = np.array([choice[e] if e // per in kept else -np.inf for e in range(n)])
    chosen = sorted(range(n), key=lambda e: (-choice[e], e))[:top]
    return [(e, s[e]) for e in chosen]


def experts(h, w, pre, ml):
    rt = ml["router"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        x = h[t:t + 1]
        for e, wt in route((x @ w[pre + "router"].T)[0], w[pre + "correction"], rt["top"], rt.get("groups")):
            out[t] += wt * (plain_unit(x, w, pre + "e%d." % e) if e < rt["experts"] else x)[0]
        if ml.get("shared"):
            g = sigmoid((x @ w[pre + "shared.sg"].T)[0, 0])
            out[t] += g * plain_unit(x, w, pre + "shared.")[0]
    return out


# ---------------------------------------------------------------------------------------------------------------- the model
class Sequence:
    """what a sequence carries from portion to portion: its length and, per layer, keys and values or latents"""

    def __init__(self, cfg):
        self.n = 0
        self.per_layer = [None] * len(cfg["layers"])


def forward(cfg, w, tokens, seq=None, layers_out=None):
    """tokens appended to seq (a new sequence if None) -> logits [T, vocab]; layers_out (a list) receives the stream after every layer"""
    seq = seq if seq is not None else Sequence(cfg)
    eps = cfg["norm"]["eps"]
    x = embed(w, tokens, seq.n)
    for i, L in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, L["mixer"]
        if L["type"] == "attention":
            y, seq.per_layer[i] = attention(x, w, p + "mix.", mx, eps, seq.n, seq.per_layer[i])
        else:
            src = mx.get("kv_from")
            y, seq.per_layer[i] = latent_attention(x, w, p + "mix.", mx, eps, seq.n, seq.per_layer[i], seq.per_layer[src] if src is not None else None)
        x = x + rms(y, w[p + "norm1"], eps)
        ml = L.get("mlp")
        if ml:
            y = gated_unit(x, w, p + "mlp.") if ml["kind"] == "dense" else experts(x, w, p + "mlp.", ml)
            x = x + rms(y, w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    seq.n += len(tokens)
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
def dense(ff=24):
    return {"kind": "dense", "ff": ff}


def moe(n=6, top=2, ff=12, identity=0, groups=None, shared=0):
    """groups: (count, keep)"""
    ml = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top}}
    if identity:
        ml["router"]["identity"] = identity
    if groups:
        ml["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        ml["shared"] = {"ff": shared}
    return ml


def layer_attention(heads=4, kv_heads=2, dim=8, coef=0.5, every=8, scale=None, mlp=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale if scale is not None else dim ** -0.5}
    if coef:
        mx["q_temp"] = {"coef": coef, "every": every}
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def layer_latent(heads=4, dim=8, vdim=12, kv_rank=16, kv_from=None, scale=None, mlp=None):
    mx = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale if scale is not None else dim ** -0.5}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mx, "mlp": mlp}


def config(layers, vocab=61, width=32, eps=1e-5):
    return {"architecture": "Gibevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def shapes_of(cfg):
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, L in enumerate(cfg["layers"]):
        p, mx, ml = "l%d." % i, L["mixer"], L.get("mlp")
        H, dn, dv = mx["heads"], mx["dim"], mx["vdim"]
        out[p + "norm1"] = (W,)
        out[p + "mix.q"], out[p + "mix.o"] = (H * dn, W), (W, H * dv)
        if L["type"] == "attention":
            out[p + "mix.k"], out[p + "mix.q.norm"], out[p + "mix.k.norm"] = (mx.get("kv_heads", H) * dn, W), (dn,), (dn,)
            out[p + "mix.g"] = (H * dv, W)
        else:
            R = mx["kv_rank"]
            if mx.get("kv_from") is None:
                out[p + "mix.dkv"], out[p + "mix.dkv.norm"] = (R, W), (R,)
            out[p + "mix.uk"], out[p + "mix.uv"], out[p + "mix.g"] = (H * dn, R), (H * dv, R), (H, W)
        if not ml:
            continue
        out[p + "norm2"] = (W,)
        if ml["kind"] == "dense":
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ml["ff"], W)
            out[p + "mlp.down"] = (W, ml["ff"])
            continue
        n = ml["router"]["experts"] + ml["router"].get("identity", 0)
        out[p + "mlp.router"], out[p + "mlp.correction"] = (n, W), (n,)
        for e in range(ml["router"]["experts"]):
            out[p + "mlp.e%d.up" % e], out[p + "mlp.e%d.down" % e] = (ml["expert"]["ff"], W), (W, ml["expert"]["ff"])
        if ml.get("shared"):
            ff = ml["shared"]["ff"]
            out[p + "mlp.shared.up"], out[p + "mlp.shared.down"], out[p + "mlp.shared.sg"] = (ff, W), (W, ff), (1, W)
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
            if last in ("norm1", "norm2"):
                a *= 0.4
        elif last == "correction":
            a = rng.uniform(-0.3, 0.1, shp)
        elif name == "embed":
            a = rng.standard_normal(shp)
        elif last == "router":
            a = 1.5 * rng.standard_normal(shp) / math.sqrt(shp[-1])
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
