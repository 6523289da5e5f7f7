"""Plain Gebuzen decoder on the CPU, one function per mechanism (test infrastructure only).

float64 numpy, loops over tokens where a mechanism is sequential; nothing is shared with the product
path.  A model is ``(config, tensors)`` as in :mod:`oracle.sudevik`.  Whole sequences go through at
once; the decoding tests compare a step at position p with row p of the whole-sequence result.
"""
import numpy as np

from oracle.sudevik import (F, Wide, linear, load_model, read_safetensors, rms_norm,  # noqa: F401
                            round_bf16, sigmoid, silu, softplus, to_bf16, widen, write_model)


# -- attention ----------------------------------------------------------------------------------
def sees(i, j, mask):
    """Does the query at position i see the key at position j?  Chunks of mask.size positions."""
    return j <= i and (not mask or i // mask["size"] == j // mask["size"])


def sink_softmax(s, sink):
    """exp(s_j) / (exp(sink) + sum exp(s))."""
    m = max(float(sink), float(np.max(s)))
    e = np.exp(s - m)
    return e / (np.exp(sink - m) + e.sum())


def attend(q, k, v, scale, mask, sink):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim], sink [H] -> [T, H, vdim]."""
    T, H, _ = q.shape
    G = k.shape[1]
    o = np.zeros((T, H, v.shape[2]), F)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, mask)]
        for h in range(H):
            g = h // (H // G)
            o[i, h] = sink_softmax(k[js, g] @ q[i, h] * scale, sink[h]) @ v[js, g]
    return o


def attention_branch(h, mc, t, pre):
    T = h.shape[0]
    H, G, D = mc["heads"], mc["kv_heads"], mc["dim"]
    q = (linear(h, t[pre + "q"]) + t[pre + "q.b"]).reshape(T, H, D)
    k = (linear(h, t[pre + "k"]) + t[pre + "k.b"]).reshape(T, G, D)
    o = attend(q, k, k, mc["scale"], mc.get("mask"), t[pre + "sink"])  # the keys are the values
    return linear(o.reshape(T, H * D), t[pre + "o"])


# -- gated linear attention -----------------------------------------------------------------------
def log_decay(h, a1, a2, bias, tau):
    """log of sigmoid(A2 A1 h + bias) ** (1 / tau)."""
    return -softplus(-(linear(linear(h, a1), a2) + bias)) / tau


def linear_attention(q, k, v, log_a, state=None):
    """q, k, log_a [T, H, dim]; v [T, H, vdim] -> o [T, H, vdim], state [H, dim, vdim]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]), F) if state is None else np.array(state, F)
    o = np.zeros(v.shape, F)
    for t in range(T):
        for h in range(H):
            S[h] = np.exp(log_a[t, h])[:, None] * S[h] + np.outer(k[t, h], v[t, h])
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def linear_branch(h, mc, t, pre, eps):
    T = h.shape[0]
    H, D, VD = mc["heads"], mc["dim"], mc["vdim"]
    q = linear(h, t[pre + "q"]).reshape(T, H, D) * D ** -0.5
    k = linear(h, t[pre + "k"]).reshape(T, H, D)
    v = linear(h, t[pre + "v"]).reshape(T, H, VD)
    la = log_decay(h, t[pre + "a1"], t[pre + "a2"], t[pre + "a2.b"], mc["tau"]).reshape(T, H, D)
    o, _ = linear_attention(q, k, v, la)
    o = rms_norm(o, t[pre + "norm"], eps).reshape(T, H * VD)
    return linear(o * silu(linear(h, t[pre + "g"])), t[pre + "o"])


# -- the model ----------------------------------------------------------------------------------
def parallel_mixer(h, mc, t, pre, eps):
    a = rms_norm(attention_branch(h, mc["left"], t, pre + "left."), t[pre + "left.out"], eps)
    b = rms_norm(linear_branch(h, mc["right"], t, pre + "right.", eps), t[pre + "right.out"], eps)
    return 0.5 * (a + b)


def dense_mlp(h, t, pre):
    return linear(np.maximum(linear(h, t[pre + "gate"]), 0.0) * linear(h, t[pre + "up"]), t[pre + "down"])


def layer_runs(cfg):
    """(layer, pass) in the order they run; pass is None outside the loop."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] + [(i, p) for p in range(loop["times"]) for i in range(a, b)] +
            [(i, None) for i in range(b, n)])


def forward(cfg, tensors, tokens, layers_out=None):
    """Logits [tokens, vocab]; `layers_out` (a list) receives the residual stream after each layer run."""
    t = tensors if isinstance(tensors, Wide) else widen(tensors)
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    first = np.array(t["embed"][np.asarray(tokens)], F)
    x = first.copy()
    for i, run in layer_runs(cfg):
        p, layer = "l%d." % i, cfg["layers"][i]
        if layer["type"] != "parallel":
            raise ValueError(layer["type"])
        if run is not None and i == cfg["loop"]["start"]:
            if run > 0:
                x = x + first
            x = x + t["loop.step"][run]
        x = x + m * parallel_mixer(rms_norm(x, t[p + "norm1"], eps), layer["mixer"], t, p + "mix.", eps)
        if layer.get("mlp"):
            x = x + m * dense_mlp(rms_norm(x, t[p + "norm2"], eps), t, p + "mlp.")
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(rms_norm(x, t["final.norm"], eps), t["head"]) * cfg["logit_scale"]


def greedy(cfg, tensors, prompt, steps):
    """`steps` tokens after `prompt`, each the first id of the largest logit."""
    ids = list(prompt)
    for _ in range(steps):
        ids.append(int(np.argmax(forward(cfg, tensors, ids)[-1])))
    return ids
