"""Small random Gebuzen models for the tests."""
import numpy as np

from oracle import sudevik as O


def layer(heads, kv_heads, dim, scale, chunk, gla_heads, gla_dim, gla_vdim, tau, ff):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if chunk:
        left["mask"] = {"size": chunk}
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": left, "right": {"heads": gla_heads, "dim": gla_dim, "vdim": gla_vdim, "tau": tau}}}


def config(vocab, width, layers, loop=None, eps=1e-6, residual_mult=0.8, logit_scale=0.5):
    c = {"architecture": "Gebuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
         "residual_mult": residual_mult, "logit_scale": logit_scale}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# sizes that fit the fast kernels; the first and the last layer alone, two in the loop
ALIGNED = config(352, 128, [
    layer(4, 2, 64, 0.12, 32, 2, 32, 48, 16.0, 192),
    layer(2, 1, 96, 0.2, 24, 4, 16, 32, 4.0, 64),
    layer(4, 4, 64, 0.1, 100, 1, 80, 64, 1.0, 0),
    layer(2, 2, 128, 0.09, 64, 2, 64, 16, 8.0, 128),
], (1, 3, 3), residual_mult=0.6, logit_scale=1.7)
# nothing is a multiple of anything; the loop is everything; a rank that is no multiple of 16
ODD = config(101, 75, [
    layer(3, 1, 21, 0.25, 7, 2, 20, 27, 16.0, 33),
    layer(2, 2, 33, 0.2, 1, 3, 13, 9, 2.5, 0),
    layer(1, 1, 10, 0.3, 0, 1, 70, 131, 30.0, 50),
], (0, 3, 2), eps=1e-4, residual_mult=1.0, logit_scale=1.0)
# larger heads, a loop at the end that is passed once, a wide rank
LARGE_HEADS = config(200, 192, [
    layer(2, 1, 200, 0.07, 33, 1, 144, 160, 16.0, 96),
    layer(10, 2, 136, 0.1, 128, 2, 160, 256, 6.0, 40),
], (1, 2, 1), residual_mult=0.5, logit_scale=0.25)
# no loop
PLAIN = config(90, 64, [layer(2, 2, 64, 0.125, 16, 2, 32, 32, 16.0, 64)] * 2)
RANKS = {"aligned": 16, "odd": 5, "large_heads": 24, "plain": 8}


def random_tensors(cfg, seed, rank=16):
    """Weights whose layers all matter: scores spread so widely that a query's few best keys hold nearly
    all the weight, so that one key too many or too few shows wherever it is; sinks from nothing to
    nearly everything; decays between fast and slow; mixers whose outputs differ in size."""
    r = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    t = {}

    def lin(name, rows, cols, gain=1.0):
        t[name] = r.normal(0, gain / np.sqrt(cols), (rows, cols))

    def norm(name, n=W):
        t[name] = 1 + 0.2 * r.normal(size=n)

    t["embed"] = r.normal(0, 1, (V, W))
    lin("head", V, W)
    norm("final.norm")
    if cfg.get("loop"):
        t["loop.step"] = r.normal(0, 0.7, (cfg["loop"]["times"], W))
    for i, l in enumerate(cfg["layers"]):
        p, a, b = "l%d." % i, l["mixer"]["left"], l["mixer"]["right"]
        norm(p + "norm1")
        m = p + "mix.left."
        for n, heads, gain in (("q", a["heads"], 2.5 / (a["scale"] * a["dim"] ** 0.5)), ("k", a["kv_heads"], 1.2)):
            lin(m + n, heads * a["dim"], W, gain)
            t[m + n + ".b"] = 0.5 * r.normal(size=heads * a["dim"])
        t[m + "sink"] = r.normal(4.0, 4.0, a["heads"])
        lin(m + "o", W, a["heads"] * a["dim"], 2.0)
        norm(m + "out")
        m = p + "mix.right."
        C = b["heads"] * b["dim"]
        for n, rows in (("q", C), ("k", C), ("v", b["heads"] * b["vdim"]), ("g", b["heads"] * b["vdim"])):
            lin(m + n, rows, W)
        lin(m + "a1", rank, W)
        lin(m + "a2", C, rank, 1.5)
        t[m + "a2.b"] = r.normal(1.0, 2.0, C)
        norm(m + "norm", b["vdim"])
        lin(m + "o", W, b["heads"] * b["vdim"], 0.5)
        norm(m + "out")
        if l["mlp"]:
            norm(p + "norm2")
            lin(p + "mlp.gate", l["mlp"]["ff"], W)
            lin(p + "mlp.up", l["mlp"]["ff"], W)
            lin(p + "mlp.down", W, l["mlp"]["ff"], 1.4)
    return {k: O.round_bf16(v.astype(np.float32)) for k, v in t.items()}
