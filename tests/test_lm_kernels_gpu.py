"""Every kernel of the floating-point decoders against the plain mechanism of the oracle, in float32
and bfloat16, at sizes that take each of its routes."""
import ctypes

import numpy as np
import pytest
import torch

from oracle import sudevik as O
from tests.sudevik_models import yarn

pytestmark = pytest.mark.gpu

DTYPES = ["f32", "bf16"]
TORCH = {"f32": torch.float32, "bf16": torch.bfloat16}
TOL = {"f32": 2e-5, "bf16": 2e-2}
I = ctypes.c_int


class AttnShape(ctypes.Structure):
    _fields_ = [(n, I) for n in ("heads", "kv_heads", "dim", "vdim", "max_step")]


class AttnMask(ctypes.Structure):
    _fields_ = [("window", I), ("keep_first", I), ("scale", ctypes.c_float), ("sink", I), ("chunk", I),
                ("sinks", ctypes.c_void_p)]


class DeltaShape(ctypes.Structure):
    _fields_ = [(n, I) for n in ("heads", "kv_heads", "dim", "vdim", "taps")]


def call(name, *args):
    from lightseq_amd import lib
    conv = []
    for a in args:
        if isinstance(a, torch.Tensor):
            conv.append(a.data_ptr())
        elif isinstance(a, ctypes.Structure):
            conv.append(ctypes.addressof(a))
        else:
            conv.append(a)
    lib.call(name, *conv, lib.current_stream())
    torch.cuda.synchronize()


def dev(a, dt="f32"):
    return torch.from_numpy(np.ascontiguousarray(a, np.float32)).cuda().to(TORCH[dt]).contiguous()


def ints(a):
    return torch.tensor(np.ascontiguousarray(a, np.int32)).cuda()


def rounded(a, dt):
    a = np.asarray(a, np.float32)
    return (O.round_bf16(a) if dt == "bf16" else a).astype(np.float64)


def host(t):
    return t.float().cpu().numpy().astype(np.float64)


def close(got, want, dt, what="", scale=None):
    scale = np.abs(want).max() if scale is None else scale
    err = np.abs(got - want).max() / max(scale, 1e-30)
    assert np.isfinite(got).all() and err < TOL[dt], "%s: error %.3g of %.3g" % (what, err, scale)


def rng(seed=0):
    return np.random.default_rng(seed)


# -- products -------------------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("m,n,k,split", [
    (1, 40, 64, 40), (5, 33, 48, 20), (16, 256, 512, 250), (40, 64, 1024, 64), (64, 100, 72, 64),
    (65, 128, 64, 128), (130, 200, 128, 190), (257, 96, 192, 96), (300, 50, 27, 44), (3, 70, 75, 70),
    (20, 16400, 72, 16400), (50, 16500, 64, 16487), (32, 700, 2056, 690), (7, 50, 1024, 50), (2048, 2048, 256, 2048), (2100, 2080, 128, 2072),
])
def test_gemm(dt, m, n, k, split):
    r = rng(m * n + k)
    a, w = rounded(r.normal(size=(m, k)), dt), rounded(r.normal(size=(n, k)), dt)
    want = a @ w.T
    ldc = (split + 7) // 8 * 8
    c = torch.zeros(m, ldc, dtype=TORCH[dt], device="cuda")
    c2 = torch.zeros(m, max(n - split, 1), device="cuda")
    call("lsh_lm_gemm_" + dt, dev(a, dt), k, dev(w, dt), c, ldc, c2, n - split, split, m, n, k)
    close(host(c)[:, :split], want[:, :split], dt)
    assert not host(c)[:, split:].any()
    if split < n:
        close(host(c2), want[:, split:], "f32", scale=np.abs(want).max())
    f = torch.zeros(m, n, device="cuda")
    call("lsh_lm_gemm_f32_out_" + dt, dev(a, dt), k, dev(w, dt), f, m, n, k)
    close(host(f), want, "f32")
    planes = ctypes.c_int(0)
    p = torch.zeros(8, m, n, device="cuda")
    call("lsh_lm_gemm_planes_" + dt, dev(a, dt), k, dev(w, dt), p, m, n, k, 8, ctypes.addressof(planes))
    assert 1 <= planes.value <= 8 and (m > 64) <= (planes.value == 1)
    close(host(p.reshape(-1)[:planes.value * m * n].reshape(planes.value, m, n)).sum(0), want, "f32")


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("m,n,k,split", [(1, 40, 64, 40), (5, 33, 48, 20), (40, 64, 1024, 64), (130, 200, 128, 176),
                                         (300, 50, 27, 44), (50, 16500, 64, 16487), (2100, 2080, 128, 2064)])
def test_gemm_scale_and_bias(dt, m, n, k, split):
    r = rng(m * n + k)
    a, w = rounded(r.normal(size=(m, k)), dt), rounded(r.normal(size=(n, k)), dt)
    bias = np.float32(r.normal(size=n) * 10).astype(np.float64)
    ldc = (split + 7) // 8 * 8
    for scale, b in ((0.3, bias), (1.0, bias), (2.5, None)):
        want = scale * (a @ w.T) + (0 if b is None else b)
        c = torch.zeros(m, ldc, dtype=TORCH[dt], device="cuda")
        c2 = torch.zeros(m, max(n - split, 1), device="cuda")
        call("lsh_lm_gemm_epilogue_" + dt, dev(a, dt), k, dev(w, dt), c, ldc, c2, n - split, split, m, n, k, scale,
             None if b is None else dev(b))
        close(host(c)[:, :split], want[:, :split], dt)
        if split < n:
            close(host(c2), want[:, split:], "f32", scale=np.abs(want).max())


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("m,n,k", [(1, 40, 64), (20, 33, 48), (33, 64, 1024), (9, 50, 1032), (32, 200, 2048), (16, 8200, 64), (30, 8200, 72), (64, 100, 72), (65, 128, 64), (130, 200, 128),
                                   (300, 50, 27), (2100, 1040, 128), (2048, 2048, 64)])
def test_gated_product(dt, m, n, k):
    r = rng(m + n + k)
    h, w = rounded(r.normal(size=(m, k)), dt), rounded(r.normal(size=(2, n, k)) / np.sqrt(k), dt)
    g, u = h @ w[0].T, h @ w[1].T
    ldc = n + 8
    for act, f in ((0, O.silu), (1, lambda z: np.maximum(z, 0))):
        c = torch.full((m, ldc), 7.0, dtype=TORCH[dt], device="cuda")
        call("lsh_lm_gemm_gated_" + dt, dev(h, dt), k, dev(w, dt), c, ldc, m, n, k, act)
        close(host(c)[:, :n], f(g) * u, dt)
        assert (host(c)[:, n:] == 7).all()


# -- routing and experts --------------------------------------------------------------------------
@pytest.mark.parametrize("tokens,experts,top", [(1, 1, 1), (37, 5, 3), (64, 64, 8), (9, 200, 17), (300, 513, 2),
                                                (513, 16, 2), (1001, 200, 5), (700, 600, 3)])
def test_route(tokens, experts, top):
    check_route(tokens, experts, top, None, 0)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("tokens,experts,top,width", [(1, 1, 1, 64), (37, 5, 3, 75), (64, 70, 8, 1024), (9, 200, 17, 40),
                                                      (3, 513, 2, 136)])
def test_router(dt, tokens, experts, top, width):
    check_route(tokens, experts, top, dt, width)


def check_route(tokens, experts, top, dt, width):
    """The choice from given logits, or (dt) from the rows and the router's weights."""
    r = rng(tokens)
    z = r.normal(size=(tokens, experts)).astype(np.float32)
    z[:, experts // 2] = z[:, 0]  # equal logits
    bias = (r.integers(-4, 5, experts) * 0.25).astype(np.float32)
    bias[experts // 2] = bias[0]
    w = torch.zeros(tokens, top, device="cuda")
    count, lst = ints(np.zeros(experts)), ints(np.full((experts, tokens), -1))
    if dt is None:
        call("lsh_lm_moe_route", dev(z), dev(bias), w, count, lst, tokens, experts, top)
    else:
        # small integers: every order of addition gives the same logits, equal ones included
        h, wr = r.integers(-2, 3, (tokens, width)), r.integers(-2, 3, (experts, width))
        wr[experts // 2] = wr[0]
        z = (h @ wr.T).astype(np.float32)
        call("lsh_lm_moe_router_" + dt, dev(h, dt), dev(wr, dt), dev(bias), w, count, lst, tokens, width, experts, top)
    w, count, lst = host(w), count.cpu().numpy(), lst.cpu().numpy()
    seen = {}
    for e in range(experts):
        for x in lst[e, :count[e]]:
            seen[x] = e
        assert (lst[e, count[e]:] == -1).all()
    assert len(seen) == tokens * top == count.sum()
    for t in range(tokens):
        chosen, want = O.route((z[t] + bias).astype(np.float32).astype(np.float64), top)
        assert [seen[t * top + j] for j in range(top)] == chosen
        assert np.allclose(w[t], want, atol=1e-6)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("tokens,experts,top,width,ff", [
    (1, 6, 2, 64, 64), (20, 12, 3, 96, 40), (50, 3, 1, 27, 9), (400, 4, 2, 128, 192), (700, 2, 1, 64, 72),
    (900, 3, 3, 192, 64), (300, 2, 2, 51, 33), (33, 1, 1, 64, 32), (200, 70, 1, 64, 64),
])
def test_experts(dt, tokens, experts, top, width, ff):
    r = rng(tokens + ff)
    h = rounded(r.normal(size=(tokens, width)), dt)
    up = rounded(r.normal(size=(experts, 2, ff, width)) / np.sqrt(width), dt)
    down = rounded(r.normal(size=(experts, width, ff)) / np.sqrt(ff), dt)
    # an uneven choice that leaves the last expert idle where it can
    live = max(experts - 1, top)
    lists = [[] for _ in range(experts)]
    choice = np.zeros((tokens, top), int)
    for t in range(tokens):
        p = np.arange(live, 0, -1.0)
        choice[t] = r.choice(live, top, replace=False, p=p / p.sum())
        for j in range(top):
            lists[choice[t, j]].append(t * top + j)
    arr = np.full((experts, tokens), -1)
    for e, x in enumerate(lists):
        arr[e, :len(x)] = r.permutation(x)
    count = ints([len(x) for x in lists])
    act = torch.zeros(tokens * top, ff, dtype=TORCH[dt], device="cuda")
    out = torch.zeros(tokens * top, width, dtype=TORCH[dt], device="cuda")
    call("lsh_lm_moe_up_" + dt, dev(h, dt), dev(up, dt), act, count, ints(arr), tokens, top, experts, width, ff)
    call("lsh_lm_moe_down_" + dt, act, dev(down, dt), out, count, ints(arr), tokens, top, experts, width, ff)
    want_a = np.stack([O.silu(h[i // top] @ up[e, 0].T) * (h[i // top] @ up[e, 1].T)
                       for i, e in enumerate(choice.reshape(-1))])
    close(host(act), want_a, dt, "up")
    want = np.stack([host(act)[i] @ down[e].T for i, e in enumerate(choice.reshape(-1))])
    close(host(out), want, dt, "down")


# -- the residual stream --------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("width", [64, 75, 1024, 1030, 3000, 8192])
def test_norm(dt, width):
    r = rng(width)
    rows, parts, eps = 7, 3, 1e-3
    x = r.normal(size=(rows, width)) + 3
    w = [1 + 0.3 * r.normal(size=width) for _ in range(2)]
    b = [r.normal(size=width) for _ in range(2)]
    f = lambda a: np.asarray(a, np.float32).astype(np.float64)  # noqa: E731
    x, w, b = f(x), [f(v) for v in w], [f(v) for v in b]
    if width % 4 and width > 4096:
        return
    # planes of partial sums, no post-norm
    y = f(r.normal(size=(parts, rows, width)))
    dx, h = dev(x), torch.zeros(rows, width, dtype=TORCH[dt], device="cuda")
    counts = ints(np.full(9, 5))
    call("lsh_lm_norm_" + dt, dx, dev(y), 1, parts, rows * width, width, None, None, None, dev(w[1]), dev(b[1]),
         h, rows, width, eps, None, None, 0, None, counts, 8)
    close(host(dx), x + y.sum(0), "f32")
    close(host(h), O.layer_norm(x + y.sum(0), w[1], b[1], eps), dt)
    assert counts.tolist() == [0] * 8 + [5]
    # weighted parts of a row with a post-norm, then no output norm
    y2 = rounded(r.normal(size=(rows, parts, width)), dt)
    wt = f(r.uniform(size=(rows, parts)))
    dx = dev(x)
    call("lsh_lm_norm_" + dt, dx, dev(y2, dt), 0, parts, width, parts * width, dev(wt), dev(w[0]), dev(b[0]),
         None, None, None, rows, width, eps, None, None, 0, None, None, 0)
    want = x + O.layer_norm((y2 * wt[..., None]).sum(1), w[0], b[0], eps)
    close(host(dx), want, "f32")
    # from the embedding table, then rows picked out of the stream
    table = rounded(r.normal(size=(11, width)), dt)
    ids = r.integers(0, 11, rows)
    call("lsh_lm_norm_" + dt, dx, None, 1, 0, 0, 0, None, None, None, dev(w[0]), dev(b[0]), h, rows, width, eps,
         ints(ids), dev(table, dt), 11, None, None, 0)
    assert np.array_equal(host(dx), table[ids])
    close(host(h), O.layer_norm(table[ids], w[0], b[0], eps), dt)
    pick = [6, 0, 3]
    call("lsh_lm_norm_" + dt, dx, None, 1, 0, 0, 0, None, None, None, dev(w[1]), dev(b[1]), h, 3, width, eps,
         None, None, 0, ints(pick), None, 0)
    close(host(h)[:3], O.layer_norm(table[ids][pick], w[1], b[1], eps), dt)


class Part(ctypes.Structure):
    _fields_ = [("y", ctypes.c_void_p), ("parts", I), ("part_stride", ctypes.c_int64), ("row_stride", ctypes.c_int64),
                ("weight", ctypes.c_void_p), ("post_w", ctypes.c_void_p), ("post_b", ctypes.c_void_p)]


class Residual(ctypes.Structure):
    _fields_ = [("part", Part * 2), ("y_is_float", I), ("post_rms", I), ("norm_rms", I), ("scale", ctypes.c_float),
                ("norm_w", ctypes.c_void_p), ("norm_b", ctypes.c_void_p), ("inject_ids", ctypes.c_void_p),
                ("inject_vec", ctypes.c_void_p)]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("width", [64, 75, 1024, 1030, 3000, 8192])
def test_residual_with_two_summands(dt, width):
    r = rng(width)
    rows, eps, scale = 7, 1e-3, 0.35
    f = lambda a: np.asarray(a, np.float32).astype(np.float64)  # noqa: E731
    x = f(r.normal(size=(rows, width)) + 3)
    w = [f(1 + 0.3 * r.normal(size=width)) for _ in range(3)]
    table, ids = rounded(r.normal(size=(11, width)), dt), r.integers(0, 11, rows)
    vec = f(r.normal(size=width))
    if width % 4 and width > 4096:
        return
    dw, dtab, dids, dvec = [dev(v) for v in w], dev(table, dt), ints(ids), dev(vec)
    h = torch.zeros(rows, width, dtype=TORCH[dt], device="cuda")
    # planes of both, each normed by itself; then the embedding again, a vector, and the norm
    y = [f(r.normal(size=(n, rows, width)) * s) for n, s in ((3, 1.0), (2, 30.0))]
    dy, dx = [dev(v) for v in y], dev(x)
    d = Residual(y_is_float=1, post_rms=1, norm_rms=1, scale=scale, norm_w=dw[2].data_ptr(),
                 inject_ids=dids.data_ptr(), inject_vec=dvec.data_ptr())
    for i in range(2):
        d.part[i] = Part(dy[i].data_ptr(), len(y[i]), rows * width, width, None, dw[i].data_ptr(), None)
    call("lsh_lm_residual_" + dt, dx, d, h, rows, width, eps, None, dtab, 11)
    want = x + scale * sum(O.rms_norm(y[i].sum(0), w[i], eps) for i in range(2)) + table[ids] + vec
    close(host(dx), want, "f32")
    close(host(h), O.rms_norm(want, w[2], eps), dt)
    # one summand in the activations' type, no norm of its own, no output
    y1 = rounded(r.normal(size=(rows, width)), dt)
    dy1, dx = dev(y1, dt), dev(x)
    d = Residual(scale=scale)
    d.part[0] = Part(dy1.data_ptr(), 1, 0, width, None, None, None)
    call("lsh_lm_residual_" + dt, dx, d, None, rows, width, eps, None, None, 0)
    close(host(dx), x + scale * y1, "f32")
    # from the embedding, with the vector
    d = Residual(norm_rms=1, scale=1.0, norm_w=dw[0].data_ptr(), inject_vec=dvec.data_ptr())
    call("lsh_lm_residual_" + dt, dx, d, h, rows, width, eps, dids, dtab, 11)
    close(host(dx), table[ids] + vec, "f32")
    close(host(h), O.rms_norm(table[ids] + vec, w[0], eps), dt)


# -- attention ------------------------------------------------------------------------------------
def cos_sin(rot, n):
    f, m = O.rope_frequencies(rot)
    a = np.arange(n)[:, None] * f
    return np.stack([m * np.cos(a), m * np.sin(a)], -1)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D,VD,rot", [
    (4, 2, 64, 64, {"base": 1e4, "dims": 64}), (3, 1, 20, 27, {"base": 300.0, "dims": 14}),
    (2, 2, 129, 200, yarn(1e5, 128, 3.0, 32, 8.0, 1.0)), (6, 3, 96, 33, None), (1, 1, 256, 256, yarn(1e4, 256, 2.0, 64, 9.0, 2.0)),
])
def test_attn_prepare(dt, H, G, D, VD, rot):
    from lightseq_amd import lib
    r = rng(D)
    rows, S, slots, eps = 9, 50, 3, 1e-5
    qc, kc, vc = 4, 4 + H * D, 4 + H * D + G * D
    proj = rounded(r.normal(size=(rows, vc + G * VD + 3)), dt)
    qn, kn = [np.float32(1 + 0.3 * r.normal(size=D)).astype(np.float64) for _ in range(2)]
    slot = r.integers(0, slots, rows)
    pos = r.permutation(S)[:rows]
    L = lib.load()
    dp, vp = L.lsh_lm_attn_pad(D), L.lsh_lm_attn_pad(VD)
    kcache = torch.full((slots, G, S, dp), 7.0, dtype=TORCH[dt], device="cuda")
    vcache = torch.full((slots, G, S, vp), 7.0, dtype=TORCH[dt], device="cuda")
    q = torch.full((rows, H, dp), 7.0, dtype=TORCH[dt], device="cuda")
    table = dev(cos_sin(rot, S)) if rot else None
    pairs = rot["dims"] // 2 if rot else 0
    sh = AttnShape(H, G, D, VD, S)
    args = lambda kcol: ("lsh_lm_attn_prepare_" + dt, dev(proj, dt), proj.shape[1], qc, kcol, vc, dev(qn), dev(kn),  # noqa: E731
                         eps, table, pairs, q, kcache, vcache, ints(slot), ints(pos), rows, sh)
    call(*args(-1))  # no keys of its own: the caches stay as they are
    assert (host(kcache) == 7).all() and (host(vcache) == 7).all()
    call(*args(kc))
    wq = O.rotate(O.rms_norm(proj[:, qc:qc + H * D].reshape(rows, H, D), qn, eps), pos, rot)
    wk = O.rotate(O.rms_norm(proj[:, kc:kc + G * D].reshape(rows, G, D), kn, eps), pos, rot)
    wv = proj[:, vc:vc + G * VD].reshape(rows, G, VD)
    close(host(q)[..., :D], wq, dt)
    assert not host(q)[..., D:].any()
    for i in range(rows):
        close(host(kcache)[slot[i], :, pos[i], :D], wk[i], dt)
        close(host(vcache)[slot[i], :, pos[i], :VD], wv[i], dt)
        assert not host(kcache)[slot[i], :, pos[i], D:].any() and not host(vcache)[slot[i], :, pos[i], VD:].any()
    written = np.zeros((slots, S), bool)
    written[slot, pos] = True
    assert (host(kcache).transpose(0, 2, 1, 3)[~written] == 7).all()


def attend_one(q, k, v, i, scale, window, keep, sink, chunk=0, logit=0.0):
    js = [j for j in range(i + 1) if j < keep or
          ((window <= 0 or i - j < window) and (chunk <= 0 or i // chunk == j // chunk))]
    s = k[js] @ q * scale
    m = max(s.max(), logit)
    e = np.exp(s - m)
    return (e / (e.sum() + (np.exp(logit - m) if sink else 0))) @ v[js]


def attention_case(dt, H, G, D, VD, spans, S, window, keep, sink=1, gate=True, seed=0, scale=None, chunk=0,
                   sinks=None, same=False):
    """spans: (pos0, n) per sequence.  One key per query position is made to stand out: the oldest
    kept one, the one just inside and the one just outside the window (the chunk) in turn."""
    from lightseq_amd import lib
    r = rng(seed + D + window)
    scale = scale or 1.5 / np.sqrt(D)
    L = lib.load()
    dp, vp = L.lsh_lm_attn_pad(D), L.lsh_lm_attn_pad(VD)
    slots = len(spans) + 1
    order = r.permutation(slots)[:len(spans)]
    rows = sum(n for _, n in spans)
    gc, ld = 8, 8 + H * VD + (-(8 + H * VD)) % 4
    kc = torch.full((slots, G, S, dp), float("nan"), dtype=TORCH[dt], device="cuda")
    vc = torch.full((slots, G, S, vp), float("nan"), dtype=TORCH[dt], device="cuda")
    q = np.zeros((rows, H, dp))
    q[..., :D] = rounded(r.normal(size=(rows, H, D)), dt)
    proj = rounded(r.normal(size=(rows, ld)), dt)
    want = np.zeros((rows, H, VD))
    meta, row, qpos = [], 0, []
    keys = []
    for (p0, n), sl in zip(spans, order):
        T = p0 + n
        k, v = np.zeros((G, T, dp)), np.zeros((G, T, vp))
        k[..., :D] = r.normal(size=(G, T, D))
        v[..., :VD] = r.normal(size=(G, T, VD))
        if same:
            v = k
        for t in range(n):
            i = p0 + t
            for g in range(G):
                far = [keep - 1, keep, i - window + 1, i - window, 0, i][(t + g) % 6]
                if chunk:
                    far = [i - i % chunk, i - i % chunk - 1, 0, i][(t // 3 + g) % 4]
                if 0 <= far <= i and far < T and t % 3 == 0:
                    q[row + t, g * (H // G), :D] = rounded(3.0 * k[g, far, :D] / np.linalg.norm(k[g, far, :D])
                                                          / scale / 2, dt)
        k, v = rounded(k, dt), rounded(v, dt)
        keys.append((k, v))
        kc[sl, :, :T] = dev(k, dt)
        if not same:
            vc[sl, :, :T] = dev(v, dt)
        meta.append((row, n, p0, sl))
        qpos += [(sl, p0 + t) for t in range(n)]
        row += n
    for (r0, n, p0, sl), (k, v) in zip(meta, keys):
        for t in range(n):
            for h in range(H):
                g = h // (H // G)
                want[r0 + t, h] = attend_one(q[r0 + t, h], k[g], v[g][:, :VD], p0 + t, scale, window, keep, sink, chunk,
                                             sinks[h] if sinks is not None else 0.0)
    if gate:
        want *= O.sigmoid(proj[:, gc:gc + H * VD].reshape(rows, H, VD))
    sh, mask = AttnShape(H, G, D, VD, S), AttnMask(window, keep, scale, sink, chunk)
    if sinks is not None:
        mask.device_sinks = dev(sinks)  # lives as long as the mask
        mask.sinks = mask.device_sinks.data_ptr()
    out = torch.zeros(rows, H * VD, dtype=TORCH[dt], device="cuda")
    head = (dev(q, dt), kc, kc if same else vc, dev(proj, dt), ld, gc if gate else -1, out)
    return head, sh, mask, meta, qpos, want.reshape(rows, -1), out


PREFILL = [
    # H, G, D, VD, spans, window, keep
    (4, 2, 64, 64, [(0, 200)], 40, 6), (2, 1, 96, 96, [(0, 1), (0, 130), (0, 64)], 64, 0),
    (3, 1, 20, 27, [(0, 70), (0, 3)], 7, 2), (2, 2, 128, 96, [(37, 90), (100, 2), (0, 129)], 33, 70),
    (1, 1, 200, 256, [(5, 60)], 0, 0), (2, 1, 33, 130, [(300, 5), (0, 300)], 1, 1),
    (2, 1, 64, 128, [(250, 64), (63, 65)], 128, 65), (1, 1, 130, 40, [(0, 150)], 1000, 3),
    (6, 2, 96, 40, [(128, 128)], 65, 129),
]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(PREFILL)))
def test_attn_prefill(dt, case):
    H, G, D, VD, spans, window, keep = PREFILL[case]
    for sink in (1, 0):
        head, sh, mask, meta, _, want, out = attention_case(dt, H, G, D, VD, spans, 320, window, keep, sink,
                                                            gate=bool(sink) or case % 2 == 0)
        call("lsh_lm_attn_prefill_" + dt, *head, ints(meta), len(meta), max(m[1] for m in meta), sh, mask)
        close(host(out), want, dt)


DECODE = [
    # H, G, D, VD, positions, window, keep
    (4, 2, 64, 64, [0, 1, 39, 40, 41, 300], 40, 6), (6, 1, 96, 96, [5, 299], 0, 0),
    (3, 1, 20, 27, [6, 7, 8, 9, 200], 7, 2), (9, 1, 128, 200, [318, 17], 100, 60),
    (2, 2, 256, 40, [0, 255, 256, 257], 256, 1), (1, 1, 33, 256, [50], 1, 3),
    (5, 1, 64, 96, [1500, 1023, 1024, 3, 2000], 1024, 5), (16, 2, 128, 128, [2047, 100], 0, 0),
    (2, 1, 64, 64, [5000, 1100, 2303], 0, 0), (1, 1, 96, 128, [4100, 2], 3000, 7),
]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(DECODE)))
def test_attn_decode(dt, case):
    from lightseq_amd import lib
    H, G, D, VD, positions, window, keep = DECODE[case]
    for sink in (1, 0):
        S = max(positions) + 5
        head, sh, mask, meta, qpos, want, out = attention_case(
            dt, H, G, D, VD, [(p, 1) for p in positions], S, window, keep, sink, gate=bool(sink))
        rows = len(positions)
        ws = torch.empty(lib.load().lsh_lm_attn_decode_workspace(rows, ctypes.addressof(sh)), device="cuda")
        for max_len in (max(positions) + 1, S):
            out.zero_()
            call("lsh_lm_attn_decode_" + dt, *head, ints([s for s, _ in qpos]), ints([p for _, p in qpos]), rows,
                 max_len, ws, sh, mask)
            close(host(out), want, dt)


# chunks, a logit per sink, values that are the keys
CHUNKED = [
    # H, G, D, VD, spans, window, keep, chunk, same
    (4, 2, 64, 64, [(0, 200)], 0, 0, 48, True), (2, 1, 96, 96, [(0, 1), (0, 130), (0, 64)], 0, 0, 64, True),
    (3, 1, 20, 27, [(0, 70), (0, 3)], 0, 2, 7, False), (2, 2, 128, 128, [(37, 90), (100, 2), (0, 129)], 0, 0, 33, True),
    (1, 1, 200, 256, [(5, 60)], 20, 0, 50, False), (2, 1, 33, 33, [(298, 5), (0, 300)], 0, 0, 1, True),
    (6, 2, 64, 64, [(250, 64), (63, 65), (127, 2)], 0, 0, 128, True), (1, 1, 250, 250, [(0, 150)], 0, 3, 1000, True),
    (2, 2, 96, 40, [(128, 128)], 65, 5, 100, False),
]


def sink_logits(H, case):
    """Among them one that takes nearly everything and one that takes nearly nothing."""
    z = rng(case).normal(size=H).astype(np.float32)
    z[0] = [6.0, -40.0, 3.0][case % 3]
    return z


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(CHUNKED)))
def test_attn_prefill_chunked(dt, case):
    H, G, D, VD, spans, window, keep, chunk, same = CHUNKED[case]
    for sinks in (sink_logits(H, case), None):
        head, sh, mask, meta, _, want, out = attention_case(dt, H, G, D, VD, spans, 320, window, keep, gate=case % 2 == 0,
                                                            chunk=chunk, sinks=sinks, same=same)
        call("lsh_lm_attn_prefill_" + dt, *head, ints(meta), len(meta), max(m[1] for m in meta), sh, mask)
        close(host(out), want, dt)


CHUNKED_DECODE = [
    # H, G, D, VD, positions, window, keep, chunk, same
    (4, 2, 64, 64, [0, 1, 39, 40, 41, 79, 80, 300], 0, 0, 40, True), (6, 1, 96, 96, [5, 299], 0, 0, 300, True),
    (3, 1, 20, 27, [6, 7, 8, 13, 14, 200], 0, 2, 7, False), (9, 1, 128, 128, [318, 17], 0, 0, 100, True),
    (2, 2, 256, 256, [0, 255, 256, 257], 0, 1, 256, True), (2, 1, 33, 33, [50], 0, 0, 1, True),
    (16, 2, 128, 128, [2047, 100, 2048, 4095], 0, 0, 2048, True), (2, 1, 64, 96, [5000, 1100, 2303], 0, 0, 4000, False),
    (1, 1, 96, 96, [3000, 2, 2999], 0, 7, 3000, True),
]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(CHUNKED_DECODE)))
def test_attn_decode_chunked(dt, case):
    from lightseq_amd import lib
    H, G, D, VD, positions, window, keep, chunk, same = CHUNKED_DECODE[case]
    S = max(positions) + 5
    head, sh, mask, meta, qpos, want, out = attention_case(
        dt, H, G, D, VD, [(p, 1) for p in positions], S, window, keep, gate=False, chunk=chunk,
        sinks=sink_logits(H, case), same=same)
    rows = len(positions)
    ws = torch.empty(lib.load().lsh_lm_attn_decode_workspace(rows, ctypes.addressof(sh)), device="cuda")
    call("lsh_lm_attn_decode_" + dt, *head, ints([s for s, _ in qpos]), ints([p for _, p in qpos]), rows, S, ws, sh,
         mask)
    close(host(out), want, dt)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(CHUNKED_DECODE)))
def test_attn_decode_append(dt, case):
    """The position's own key comes with the projection and is in the cache afterwards."""
    from lightseq_amd import lib
    from lightseq_amd.lib import LSHError
    H, G, D, VD, positions, window, keep, chunk, same = CHUNKED_DECODE[case]
    S, rows = max(positions) + 5, len(positions)
    (q, kc, *_, out), sh, mask, meta, qpos, want, out = attention_case(
        dt, H, G, D, D, [(p, 1) for p in positions], S, window, keep, gate=False, chunk=chunk,
        sinks=sink_logits(H, case), same=True)
    slots, pos = [s for s, _ in qpos], [p for _, p in qpos]
    ld, qc, kcol = 16 + (H + G) * D + (-(H + G) * D) % 8, 16 + G * D, 8
    proj = np.zeros((rows, ld))
    proj[:, qc:qc + H * D] = host(q)[..., :D].reshape(rows, -1)
    before = host(kc)
    for i in range(rows):
        proj[i, kcol:kcol + G * D] = before[slots[i], :, pos[i], :D].reshape(-1)
        kc[slots[i], :, pos[i]] = float("nan")
    ws = torch.empty(lib.load().lsh_lm_attn_decode_workspace(rows, ctypes.addressof(sh)), device="cuda")
    args = ("lsh_lm_attn_decode_append_" + dt, dev(proj, dt), ld, qc, kcol, kc, out, ints(slots), ints(pos), rows, S, ws,
            sh, mask)
    if D not in (64, 96, 128, 256):
        with pytest.raises(LSHError, match="need padding"):
            call(*args)
        return
    call(*args)
    close(host(out), want, dt)
    assert np.array_equal(host(kc), before, equal_nan=True)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("m,n,k0,k1", [(1, 40, 64, 2048), (16, 128, 1024, 96), (33, 250, 512, 512), (64, 64, 72, 4096),
                                       (65, 48, 64, 128), (5, 30, 27, 64), (20, 16400, 64, 72)])
def test_two_products_at_once(dt, m, n, k0, k1):
    r = rng(m + k0)
    a = [rounded(r.normal(size=(m, k)), dt) for k in (k0, k1)]
    w = [rounded(r.normal(size=(n, k)), dt) for k in (k0, k1)]
    c = [torch.full((8, m, n), float("nan"), device="cuda") for _ in range(2)]
    planes = [ctypes.c_int(0), ctypes.c_int(0)]
    call("lsh_lm_gemm_planes2_" + dt, dev(a[0], dt), k0, dev(w[0], dt), c[0], k0, dev(a[1], dt), k1, dev(w[1], dt), c[1],
         k1, m, n, 8, *map(ctypes.addressof, planes))
    for i in range(2):
        got = host(c[i]).reshape(-1)[:planes[i].value * m * n].reshape(planes[i].value, m, n).sum(0)
        close(got, a[i] @ w[i].T, "f32")


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D", [(4, 2, 64), (3, 1, 20), (2, 2, 129), (1, 1, 256)])
def test_attn_prepare_without_norm_rotation_and_values(dt, H, G, D):
    from lightseq_amd import lib
    r = rng(D)
    rows, S, slots = 9, 50, 3
    qc, kc = 8, 8 + H * D
    proj = rounded(r.normal(size=(rows, kc + G * D + 4)), dt)
    slot, pos = r.integers(0, slots, rows), r.permutation(S)[:rows]
    dp = lib.load().lsh_lm_attn_pad(D)
    kcache = torch.full((slots, G, S, dp), 7.0, dtype=TORCH[dt], device="cuda")
    q = torch.full((rows, H, dp), 7.0, dtype=TORCH[dt], device="cuda")
    call("lsh_lm_attn_prepare_" + dt, dev(proj, dt), proj.shape[1], qc, kc, -1, None, None, 0.0, None, 0, q, kcache,
         None, ints(slot), ints(pos), rows, AttnShape(H, G, D, D, S))
    assert np.array_equal(host(q)[..., :D], proj[:, qc:qc + H * D].reshape(rows, H, D)) and not host(q)[..., D:].any()
    got, written = host(kcache), np.zeros((slots, S), bool)
    for i in range(rows):
        assert np.array_equal(got[slot[i], :, pos[i], :D], proj[i, kc:kc + G * D].reshape(G, D))
        assert not got[slot[i], :, pos[i], D:].any()
    written[slot, pos] = True
    assert (got.transpose(0, 2, 1, 3)[~written] == 7).all()


# -- gated delta rule -----------------------------------------------------------------------------
class Delta:
    """Random inputs of one layer for sequences of given lengths, and what the oracle makes of them."""

    def __init__(self, dt, H, G, D, VD, taps, lengths, seed=0, hard=False):
        r = rng(seed + D)
        self.dt, self.sh, self.lengths = dt, DeltaShape(H, G, D, VD, taps), lengths
        C = 2 * G * D + H * VD
        self.g_col, self.ld = C, C + H * VD + 5
        self.conv = np.float32(r.normal(0, 0.7, (C, taps))).astype(np.float64)
        self.a_log = np.float32(r.uniform(-5, 1, H)).astype(np.float64)
        self.dt_bias = np.float32(r.normal(size=H)).astype(np.float64)
        self.norm_w = np.float32(1 + 0.2 * r.normal(size=VD)).astype(np.float64)
        self.eps = 1e-5
        self.proj = [rounded(r.normal(size=(n, self.ld)), dt) for n in lengths]
        self.ba = [np.float32(r.normal(0, 3 if hard else 1, (n, 2 * H))).astype(np.float64) for n in lengths]
        if hard:  # keys that hardly change from token to token
            for p in self.proj:
                p[:, G * D:2 * G * D] = rounded(p[:1, G * D:2 * G * D] + 0.02 * p[:, G * D:2 * G * D], dt)
        self.o, self.out, self.q, self.k, self.v, self.beta, self.g, self.S = ([] for _ in range(8))
        for p, ba in zip(self.proj, self.ba):
            n = len(p)
            y = O.silu(O.short_conv(p[:, :C], self.conv))
            q = O.unit(y[:, :G * D].reshape(n, G, D)) * D ** -0.5
            k = O.unit(y[:, G * D:2 * G * D].reshape(n, G, D))
            v = y[:, 2 * G * D:].reshape(n, H, VD)
            beta = O.sigmoid(ba[:, :H])
            lg = -np.exp(self.a_log) * O.softplus(ba[:, H:] + self.dt_bias)
            o, S = O.delta_rule(q, k, v, np.exp(lg), beta)
            gate = p[:, self.g_col:self.g_col + H * VD].reshape(n, H, VD)
            for lst, x in ((self.q, q), (self.k, k), (self.v, v), (self.beta, beta), (self.g, lg), (self.o, o),
                           (self.S, S), (self.out, O.rms_norm(o, self.norm_w, self.eps) * O.silu(gate))):
                lst.append(x)

    def device(self, slots):
        sh = self.sh
        C = 2 * sh.kv_heads * sh.dim + sh.heads * sh.vdim
        self.ring = torch.full((slots, sh.taps, C), float("nan"), dtype=TORCH[self.dt], device="cuda")
        self.state = torch.full((slots, sh.heads, sh.dim, sh.vdim), float("nan"), device="cuda")
        self.consts = [dev(x) for x in (self.conv, self.a_log, self.dt_bias)]

    def run_spans(self, cuts, kernel):
        """cuts: (sequence, slot, first, last) of one batch; returns o and the gated output."""
        sh, dt = self.sh, self.dt
        meta, row = [], 0
        for i, slot, a, b in cuts:
            meta.append((row, b - a, a, slot))
            row += b - a
        proj = dev(np.concatenate([self.proj[i][a:b] for i, _, a, b in cuts]), dt)
        ba = dev(np.concatenate([self.ba[i][a:b] for i, _, a, b in cuts]))
        z = lambda *s, d=torch.float32: torch.full(s, float("nan"), dtype=d, device="cuda")  # noqa: E731
        q, k = z(row, sh.kv_heads, sh.dim), z(row, sh.kv_heads, sh.dim)
        v = z(row, sh.heads, sh.vdim, d=TORCH[dt])
        lg, be, o = z(row, sh.heads), z(row, sh.heads), z(row, sh.heads, sh.vdim)
        out = z(row, sh.heads, sh.vdim, d=TORCH[dt])
        n, mx, sp = len(meta), max(m[1] for m in meta), ints(meta)
        call("lsh_lm_delta_prepare_" + dt, proj, self.ld, ba, *self.consts, self.ring, q, k, v, lg, be, sp, n, mx, sh)
        if kernel == "scan":
            call("lsh_lm_delta_scan_" + dt, q, k, v, lg, be, self.state, o, sp, n, sh)
        else:
            from lightseq_amd import lib
            ws = z(lib.load().lsh_lm_delta_chunked_workspace(row, n, ctypes.addressof(sh)))
            call("lsh_lm_delta_chunked_" + dt, q, k, v, lg, be, self.state, o, ws, sp, n, mx, row, sh)
        call("lsh_lm_delta_gated_norm_" + dt, o, proj, self.ld, self.g_col, dev(self.norm_w), self.eps, out, row, sh)
        cat = lambda lst: np.concatenate([lst[i][a:b] for i, _, a, b in cuts])  # noqa: E731
        close(host(q), cat(self.q), "f32", "q")
        close(host(k), cat(self.k), "f32", "k")
        close(host(v), cat(self.v), dt, "v")
        close(host(lg), cat(self.g), "f32", "log decay")
        close(host(be), cat(self.beta), "f32", "beta")
        close(host(o), cat(self.o), dt, "o")
        close(host(out), cat(self.out), dt, "gated")

    def step(self, rows):
        """rows: (sequence, slot, position), one token each."""
        sh, dt = self.sh, self.dt
        proj = dev(np.stack([self.proj[i][p] for i, _, p in rows]), dt)
        ba = dev(np.stack([self.ba[i][p] for i, _, p in rows]))
        out = torch.full((len(rows), sh.heads, sh.vdim), float("nan"), dtype=TORCH[dt], device="cuda")
        call("lsh_lm_delta_step_" + dt, proj, self.ld, self.g_col, ba, *self.consts, dev(self.norm_w), self.eps,
             self.ring, self.state, out, ints([s for _, s, _ in rows]), ints([p for _, _, p in rows]), len(rows), sh)
        close(host(out), np.stack([self.out[i][p] for i, _, p in rows]), dt, "step")


DELTA = [
    # H, G, D, VD, taps
    (4, 2, 32, 48, 4), (6, 2, 21, 19, 2), (2, 1, 144, 160, 1), (1, 1, 12, 70, 5), (3, 3, 128, 128, 8), (2, 2, 256, 256, 3),
    (2, 1, 64, 30, 4), (2, 1, 80, 16, 3), (2, 1, 32, 32, 11),
]


def chunkable(sh):
    from lightseq_amd import lib
    return bool(lib.load().lsh_lm_delta_chunked_supported(ctypes.addressof(sh)))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(DELTA)))
def test_delta(dt, case):
    H, G, D, VD, taps = DELTA[case]
    lengths = [131, 64, 7, 200]
    d = Delta(dt, H, G, D, VD, taps, lengths, case)
    if not chunkable(d.sh):
        with pytest.raises(Exception, match="multiples of 16"):
            d.device(5)
            d.run_spans([(0, 0, 0, 4)], "chunked")
    for kernel in ("scan", "chunked") if chunkable(d.sh) else ("scan",):
        d.device(5)
        # whole sequences of unequal length in one batch
        d.run_spans([(0, 3, 0, 131), (1, 0, 0, 64), (2, 4, 0, 7), (3, 1, 0, 200)], kernel)
        for i, slot in ((0, 3), (1, 0), (2, 4), (3, 1)):
            close(host(d.state[slot]), d.S[i], dt, "state")
        # portions, down to one and two tokens, on slots used before
        for a, b in ((0, 2), (2, 3), (3, 66), (66, 130), (130, 131)):
            d.run_spans([(3, 3, a, b), (0, 1, a, b)], kernel)
        close(host(d.state[1]), d.S[0], dt, "state")
    # prompt, then decoding; a sequence decoded from its first token beside it
    d.device(5)
    d.run_spans([(0, 2, 0, 70)], "chunked" if chunkable(d.sh) else "scan")
    for t in range(40):
        d.step([(0, 2, 70 + t), (1, 4, t)])
    d.step([(2, 2, 0), (0, 0, 0)])  # slot 2 again, by another sequence
    d.step([(2, 2, 1)])


@pytest.mark.parametrize("kernel", ["scan", "chunked"])
def test_delta_keys_that_hardly_change(kernel):
    """The triangular system of a chunk is at its worst when all keys point one way."""
    d = Delta("f32", 2, 1, 64, 32, 4, [400], 3, hard=True)
    d.device(1)
    d.run_spans([(0, 0, 0, 400)], kernel)
    close(host(d.state[0]), d.S[0], "f32", "state")


# -- sampling -------------------------------------------------------------------------------------
class Sampler:
    def __init__(self, logits, max_step=32, lens=None):
        from lightseq_amd import lib
        self.z = dev(logits)
        self.rows, self.vocab = logits.shape
        self.max_step = max_step
        self.rng = torch.zeros(2 * self.rows, dtype=torch.int64, device="cuda")
        lib.call("lsh_rng_setup", self.rng.data_ptr(), self.rows, 5, lib.current_stream())
        self.ids = ints(np.full((self.rows, max_step), -9))
        self.last, self.len = ints(np.zeros(self.rows)), ints(lens if lens is not None else np.zeros(self.rows))
        self.pos, self.flag = ints(np.zeros(self.rows)), ints([0])

    def draw(self, topk, topp=0.0, eos=-1):
        call("lsh_lm_sample", self.z, self.rows, self.vocab, topk, topp, eos, self.rng, self.ids, self.max_step,
             self.last, self.len, self.pos, self.flag)
        return self.last.cpu().numpy()


def test_sample_greedy_takes_the_first_of_equals_and_keeps_count():
    z = np.zeros((3, 5000), np.float32)
    z[0, [17, 4000]] = 2
    z[1, 4999] = 1
    z[2] = -3
    s = Sampler(z, lens=[0, 4, 9])
    assert s.draw(1, eos=4999).tolist() == [17, 4999, 0]
    assert s.ids[0, 0] == 17 and s.ids[1, 4] == 4999 and s.ids[2, 9] == 0
    assert s.len.tolist() == [1, -5, 10] and s.pos.tolist() == [0, 4, 9] and s.flag.item() == 1
    s.draw(1, eos=4999)  # an ended row stays
    assert s.len.tolist() == [2, -5, 11] and (s.ids[1, 5:] == -9).all()


def test_sample_topk_and_topp_stay_in_their_sets_with_the_right_shares():
    r = rng(1)
    V, n = 777, 600
    row = r.normal(size=V).astype(np.float32) * 2
    order = np.argsort(-row, kind="stable")
    p = np.exp(row - row.max()).astype(np.float64)
    for topk, topp in ((5, 0.0), (0, 0.4), (0, 1.0), (1000, 0.0)):
        if topk:
            keep = order[:topk]
        else:
            c = np.cumsum(p[order]) / p.sum()
            keep = order[:min(int(np.searchsorted(c, topp)) + 1, V)]
        s = Sampler(np.tile(row, (n, 1)))
        got = s.draw(topk, topp)
        assert set(got) <= set(keep.tolist())
        top = keep[0]
        share = p[top] / p[keep].sum()
        assert abs((got == top).mean() - share) < 5 * np.sqrt(share * (1 - share) / n) + 1e-3
        assert len(set(got)) > 1
        assert s.draw(topk, topp).tolist() != got.tolist()  # the streams advance


def test_bad_arguments_are_refused():
    from lightseq_amd.lib import LSHError
    x = torch.zeros(64, device="cuda")
    with pytest.raises(LSHError, match="bad arguments"):
        call("lsh_lm_gemm_f32", x, 8, x, x, 8, None, 0, 8, 0, 8, 8)
    with pytest.raises(LSHError, match="no second output"):
        call("lsh_lm_gemm_f32", x, 8, x, x, 8, None, 0, 4, 1, 8, 8)
    with pytest.raises(LSHError, match="256"):
        call("lsh_lm_attn_prefill_f32", x, x, x, x, 8, -1, x, ints([0, 1, 0, 0]), 1, 1,
             AttnShape(1, 1, 300, 8, 8), AttnMask(0, 0, 1.0, 1))
    with pytest.raises(LSHError, match="at most 64 choices"):
        call("lsh_lm_moe_route", x, None, x, ints(np.zeros(100)), ints(np.zeros(100)), 1, 100, 65)
    with pytest.raises(LSHError, match="topp"):
        call("lsh_lm_sample", x, 1, 8, 0, 0.0, -1, x, ints([0]), 1, ints([0]), ints([0]), ints([0]), ints([0]))
