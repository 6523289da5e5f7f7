"""Small random Sudevik models for the tests: configurations, weights, and a runner that feeds a
model's step interface."""
import numpy as np

from oracle import sudevik as O


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def attention(heads, kv_heads, dim, vdim, scale, rot=None, mask=None, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot:
        m["rot"] = rot
    if mask:
        m["mask"] = mask
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def delta(heads, kv_heads, dim, vdim, conv, mlp=None):
    return {"type": "delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                                                   "vdim": vdim, "conv": conv}}


def yarn(base, dims, factor, original, fast, slow):
    return {"base": base, "dims": dims,
            "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}


def config(vocab, width, layers, eps=1e-6):
    return {"architecture": "Sudevik", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": layers}


# sizes that fit the fast kernels
ALIGNED = config(352, 128, [
    delta(4, 2, 32, 48, 4, moe(10, 2, 64)),
    attention(4, 2, 64, 32, 0.3, yarn(10000.0, 64, 4.0, 128, 16.0, 2.0),
              {"size": 24, "keep_first": 3}, mlp=moe(6, 1, 128)),
    delta(2, 2, 80, 16, 3, None),
    attention(4, 2, 64, 32, 0.45, yarn(10000.0, 64, 4.0, 128, 16.0, 2.0),
              {"size": 70, "keep_first": 9}, kv_from=1, mlp=moe(10, 3, 64)),
])
# nothing is a multiple of anything; branches that may be absent are
ODD = config(101, 75, [
    attention(3, 1, 20, 27, 0.4, {"base": 500.0, "dims": 14}, {"size": 7, "keep_first": 0},
              mlp=moe(5, 3, 23)),
    delta(6, 2, 21, 19, 2, moe(7, 1, 9)),
    attention(2, 2, 33, 40, 0.3, None, {"size": 1, "keep_first": 2}, mlp=None),
    delta(1, 1, 12, 70, 5, moe(3, 3, 33)),
    attention(3, 1, 20, 27, 0.6, {"base": 500.0, "dims": 14}, None, kv_from=0, mlp=moe(4, 2, 12)),
], eps=1e-4)
# larger heads, one expert, one tap
LARGE_HEADS = config(200, 192, [
    delta(2, 1, 144, 160, 1, moe(2, 2, 96)),
    attention(10, 2, 136, 200, 0.2, yarn(1e6, 100, 8.0, 64, 32.0, 1.0),
              {"size": 33, "keep_first": 40}, mlp=moe(1, 1, 40)),
])


def random_tensors(cfg, seed):
    """Weights whose layers all matter: unit-scale projections, decays between fast and slow."""
    r = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    t = {}

    def lin(name, rows, cols, gain=1.0):
        t[name] = r.normal(0, gain / np.sqrt(cols), (rows, cols))

    def norm(name, n=W, bias=True):
        t[name] = 1 + 0.2 * r.normal(size=n)
        if bias:
            t[name + ".b"] = 0.1 * r.normal(size=n)

    t["embed"] = r.normal(0, 1, (V, W))
    lin("head", V, W)
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        H, G, D, VD = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] else ()):
            norm(p + n)
        q = p + "mix."
        if l["type"] == "attention":
            lin(q + "q", H * D, W)
            norm(q + "q.norm", D, False)
            if m.get("kv_from") is None:
                lin(q + "k", G * D, W)
                lin(q + "v", G * VD, W)
                norm(q + "k.norm", D, False)
        else:
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * VD)):
                lin(q + n, rows, W)
                t[q + n + ".conv"] = r.normal(0, 0.6, (rows, m["conv"]))
            lin(q + "b", H, W)
            lin(q + "a", H, W)
            t[q + "A_log"] = r.uniform(-4, 0.5, H)
            t[q + "dt_bias"] = r.normal(-1, 1, H)
            norm(q + "norm", VD, False)
        lin(q + "g", H * VD, W)
        lin(q + "o", W, H * VD)
        if l["mlp"]:
            E, F = l["mlp"]["router"]["experts"], l["mlp"]["expert"]["ff"]
            lin(p + "mlp.router", E, W, 2.0)
            t[p + "mlp.router.b"] = 0.3 * r.normal(size=E)
            for e in range(E):
                lin(p + "mlp.e%d.gate" % e, F, W)
                lin(p + "mlp.e%d.up" % e, F, W)
                lin(p + "mlp.e%d.down" % e, W, F)
    return {k: O.round_bf16(v.astype(np.float32)) for k, v in t.items()}


class Fed:
    """A model with named sequences: feed({name: tokens}) -> {name: logits of all these tokens}."""

    def __init__(self, model):
        self.model, self.slot = model, {}

    def feed(self, batch):
        entries, n = [], 0
        for name, toks in batch.items():
            if name not in self.slot:
                self.slot[name] = self.model.open_sequence()
            entries.append((self.slot[name], list(toks)))
            n += len(toks)
        out = self.model.step(entries, range(n))
        res, at = {}, 0
        for name, toks in batch.items():
            res[name] = out[at:at + len(toks)]
            at += len(toks)
        return res

    def end(self, *names):
        for n in names:
            self.model.close_sequence(self.slot.pop(n))


def row_errors(got, want):
    """Per row: RMS difference relative to the RMS of the expected logits, means removed."""
    g = np.asarray(got, np.float64)
    d = g - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean())
