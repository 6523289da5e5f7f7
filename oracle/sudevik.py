"""Plain Sudevik decoder on the CPU, one function per mechanism (test infrastructure only).

Everything is computed in float64 numpy with explicit loops over tokens where the mechanism is
sequential; nothing is shared with the product path.  A model is ``(config, tensors)``: the parsed
config.json and a dict of float arrays.  Whole sequences go through at once; the decoding tests
compare a step at position p with row p of the whole-sequence result.
"""
import json
import math
import os

import numpy as np

F = np.float64


def read_safetensors(path):
    """name -> array (bfloat16 widened to float32); the format is read here, without a library."""
    with open(path, "rb") as f:
        raw = f.read()
    n = int.from_bytes(raw[:8], "little")
    head = json.loads(raw[8:8 + n].decode())
    out = {}
    for name, d in head.items():
        if name == "__metadata__":
            continue
        a, b = d["data_offsets"]
        buf = raw[8 + n + a:8 + n + b]
        if d["dtype"] == "BF16":
            v = (np.frombuffer(buf, np.uint16).astype(np.uint32) << 16).view(np.float32)
        elif d["dtype"] == "F32":
            v = np.frombuffer(buf, np.float32)
        elif d["dtype"] == "I32":
            v = np.frombuffer(buf, np.int32)
        else:
            raise ValueError(d["dtype"])
        out[name] = v.reshape(d["shape"])
    return out


def to_bf16(a):
    """float32 array -> uint16 words of its bfloat16 rounding (nearest even)."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7fff + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def round_bf16(a):
    return (to_bf16(a).astype(np.uint32) << 16).view(np.float32)


def write_model(path, config, tensors):
    """config.json + model.safetensors (bfloat16) in the folder `path`."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    head, blobs, at = {}, [], 0
    for name, v in tensors.items():
        b = to_bf16(v).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h + b"".join(blobs))


def load_model(path):
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return cfg, read_safetensors(os.path.join(path, "model.safetensors"))


# -- elementary functions -----------------------------------------------------------------------
def sigmoid(z):
    z = np.asarray(z, F)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def layer_norm(x, w, b, eps):
    x = np.asarray(x, F)
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w + b


def rms_norm(x, w, eps):
    x = np.asarray(x, F)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def linear(h, w):
    return h @ np.asarray(w, F).T


# -- rotation -----------------------------------------------------------------------------------
def rope_frequencies(rot):
    """(frequency per pair, factor on cos and sin)."""
    dims, base = rot["dims"], float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], F)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def turn(t):
        return dims * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo = max(math.floor(turn(sc["fast"])), 0)
    hi = min(math.ceil(turn(sc["slow"])), dims - 1)
    out = []
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f[i] / sc["factor"] * ramp + f[i] * (1 - ramp))
    return np.array(out, F), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [tokens, heads, dim]; interleaved pairs (2i, 2i+1) of the first rot.dims dimensions."""
    if not rot:
        return x
    f, m = rope_frequencies(rot)
    y = np.array(x, F)
    for t, p in enumerate(positions):
        for i in range(rot["dims"] // 2):
            c, s = m * math.cos(p * f[i]), m * math.sin(p * f[i])
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            y[t, :, 2 * i] = u * c - v * s
            y[t, :, 2 * i + 1] = v * c + u * s
    return y


# -- attention ----------------------------------------------------------------------------------
def sees(i, j, mask):
    """Does the query at position i see the key at position j?"""
    return j <= i and (i - j < mask["size"] or j < mask["keep_first"])


def sink_softmax(s):
    """exp(s_j) / (1 + sum exp(s)), the one being a sink of score 0 without a value."""
    m = max(0.0, float(np.max(s)))
    e = np.exp(s - m)
    return e / (math.exp(-m) + e.sum())


def attend(q, k, v, scale, mask):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]."""
    T, H, _ = q.shape
    G = k.shape[1]
    o = np.zeros((T, H, v.shape[2]), F)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, mask)] if mask else list(range(i + 1))
        for h in range(H):
            g = h // (H // G)
            o[i, h] = sink_softmax(k[js, g] @ q[i, h] * scale) @ v[js, g]
    return o


def attention_mixer(h, mc, t, pre, eps, kv_store):
    """kv_store: layer index -> (keys after norm and rotation, values); read and extended here."""
    T = h.shape[0]
    H, G, D, VD = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    pos = range(T)
    q = rms_norm(linear(h, t[pre + "q"]).reshape(T, H, D), t[pre + "q.norm"], eps)
    q = rotate(q, pos, mc.get("rot"))
    if mc.get("kv_from") is not None:
        k, v = kv_store[mc["kv_from"]]
    else:
        k = rms_norm(linear(h, t[pre + "k"]).reshape(T, G, D), t[pre + "k.norm"], eps)
        k = rotate(k, pos, mc.get("rot"))
        v = linear(h, t[pre + "v"]).reshape(T, G, VD)
    o = attend(q, k, v, mc["scale"], mc.get("mask"))
    gate = sigmoid(linear(h, t[pre + "g"]))
    return linear(o.reshape(T, H * VD) * gate, t[pre + "o"]), (k, v)


# -- gated delta rule ---------------------------------------------------------------------------
def short_conv(x, w):
    """Causal convolution per channel: y[t] = sum_k w[:, k] x[t - taps + 1 + k]."""
    T, C = x.shape
    taps = w.shape[1]
    xp = np.concatenate([np.zeros((taps - 1, C), F), x])
    y = np.zeros((T, C), F)
    for k in range(taps):
        y += xp[k:k + T] * w[:, k]
    return y


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta, state=None):
    """q, k [T, G, dim]; v [T, H, vdim]; g, beta [T, H] -> o [T, H, vdim], state [H, dim, vdim]."""
    T, H, VD = v.shape
    G, D = q.shape[1:]
    S = np.zeros((H, D, VD), F) if state is None else np.array(state, F)
    o = np.zeros((T, H, VD), F)
    for t in range(T):
        for h in range(H):
            c = h // (H // G)
            S[h] *= g[t, h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, c])
            S[h] += np.outer(k[t, c], u)
            o[t, h] = S[h].T @ q[t, c]
    return o, S


def delta_mixer(h, mc, t, pre, eps):
    T = h.shape[0]
    H, G, D, VD = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    proj = {n: silu(short_conv(linear(h, t[pre + n]), np.asarray(t[pre + n + ".conv"], F)))
            for n in "qkv"}
    q = unit(proj["q"].reshape(T, G, D)) * D ** -0.5
    k = unit(proj["k"].reshape(T, G, D))
    v = proj["v"].reshape(T, H, VD)
    beta = sigmoid(linear(h, t[pre + "b"]))
    g = np.exp(-np.exp(np.asarray(t[pre + "A_log"], F)) * softplus(linear(h, t[pre + "a"]) +
                                                                  t[pre + "dt_bias"]))
    o, _ = delta_rule(q, k, v, g, beta)
    o = rms_norm(o, t[pre + "norm"], eps) * silu(linear(h, t[pre + "g"])).reshape(T, H, VD)
    return linear(o.reshape(T, H * VD), t[pre + "o"])


# -- mixture of experts -------------------------------------------------------------------------
def route(z, top):
    """The `top` largest logits of one token and the soft-max over them."""
    chosen = sorted(range(len(z)), key=lambda e: (-z[e], e))[:top]
    e = np.exp(np.array([z[c] for c in chosen]) - max(z[c] for c in chosen))
    return chosen, e / e.sum()


def moe(h, fc, t, pre):
    z = linear(h, t[pre + "router"]) + t[pre + "router.b"]
    out = np.zeros((h.shape[0], h.shape[1]), F)
    for i in range(h.shape[0]):
        for e, w in zip(*route(z[i], fc["router"]["top"])):
            p = "%se%d." % (pre, e)
            out[i] += w * linear(silu(linear(h[i], t[p + "gate"])) * linear(h[i], t[p + "up"]),
                                 t[p + "down"])
    return out


# -- the model ----------------------------------------------------------------------------------
def forward(cfg, tensors, tokens, layers_out=None):
    """Logits [tokens, vocab]; `layers_out` (a list) receives the residual stream after each layer."""
    t = {n: np.asarray(v, F) for n, v in tensors.items()} if not isinstance(tensors, Wide) else tensors
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return layer_norm(x, t[name], t[name + ".b"], eps)
    x = np.array(t["embed"][np.asarray(tokens)], F)
    kv = {}
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % i
        h = norm(x, p + "norm1")
        if layer["type"] == "attention":
            y, kv[i] = attention_mixer(h, layer["mixer"], t, p + "mix.", eps, kv)
        elif layer["type"] == "delta":
            y = delta_mixer(h, layer["mixer"], t, p + "mix.", eps)
        else:
            raise ValueError(layer["type"])
        x = x + norm(y, p + "norm1b")
        if layer.get("mlp"):
            x = x + norm(moe(norm(x, p + "norm2"), layer["mlp"], t, p + "mlp."), p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(norm(x, "final.norm"), t["head"])


class Wide(dict):
    """Tensors already widened to float64 (saves the conversion in repeated calls)."""


def widen(tensors):
    return Wide((n, np.asarray(v, F)) for n, v in tensors.items())


def greedy(cfg, tensors, prompt, steps):
    """`steps` tokens after `prompt`, each the first id of the largest logit."""
    ids = list(prompt)
    for _ in range(steps):
        ids.append(int(np.argmax(forward(cfg, tensors, ids)[-1])))
    return ids
