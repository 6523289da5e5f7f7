"""The kernels of gated linear attention against the plain recurrence, in float32 and bfloat16: token by
token, in chunks, in portions, decoded, on states used before."""
import ctypes

import numpy as np
import pytest
import torch

from oracle import gebuzen as O
from tests.test_lm_kernels_gpu import DTYPES, I, TORCH, call, close, dev, host, ints, rng, rounded

pytestmark = pytest.mark.gpu


class GlaShape(ctypes.Structure):
    _fields_ = [(n, I) for n in ("heads", "dim", "vdim", "rank", "q_col", "k_col", "v_col", "g_col")] + \
               [("tau", ctypes.c_float), ("eps", ctypes.c_float)]


class Gla:
    """Random inputs of one layer for sequences of given lengths, and what the oracle makes of them.
    decay: mean of the logit that the decays are made from."""

    def __init__(self, dt, H, D, VD, rank, tau, lengths, seed=0, decay=0.0):
        r = rng(seed + D)
        f = lambda a: np.asarray(a, np.float32).astype(np.float64)  # noqa: E731
        self.dt, self.lengths = dt, lengths
        self.rank = -(-rank // 16) * 16
        up8 = lambda n: -(-n // 8) * 8  # noqa: E731
        q = 8
        k, v = q + up8(H * D), q + 2 * up8(H * D)
        g = v + up8(H * VD)
        self.ld = g + up8(H * VD)
        self.sh = GlaShape(H, D, VD, self.rank, q, k, v, g, tau, 1e-5)
        self.a2 = f(r.normal(size=(H * D, rank)) / np.sqrt(rank))
        self.bias = f(r.normal(decay, 2.0, H * D))
        self.norm = f(1 + 0.2 * r.normal(size=VD))
        self.proj = [rounded(r.normal(size=(n, self.ld)), dt) for n in lengths]
        self.low = [f(r.normal(size=(n, rank))) for n in lengths]
        self.out, self.S = [], []
        for p, low in zip(self.proj, self.low):
            n = len(p)
            cols = lambda at, w: p[:, at:at + H * w].reshape(n, H, w)  # noqa: E731
            # the first product has been made already
            la = O.log_decay(low, np.eye(rank), self.a2, self.bias, tau).reshape(n, H, D)
            o, S = O.linear_attention(cols(q, D) * D ** -0.5, cols(k, D), cols(v, VD), la)
            self.out.append(O.rms_norm(o, self.norm, 1e-5) * O.silu(cols(g, VD)))
            self.S.append(S.transpose(0, 2, 1))

    def device(self, slots):
        sh = self.sh
        pad = lambda a: np.concatenate([a, np.zeros((len(a), self.rank - a.shape[1]))], 1)  # noqa: E731
        self.weights = [dev(pad(self.a2)), dev(self.bias), dev(self.norm)]
        self.pad = pad
        self.state = torch.full((slots, sh.heads, sh.vdim, sh.dim), float("nan"), device="cuda")

    def args(self, rows):
        """rows: (sequence, positions)"""
        proj = np.concatenate([self.proj[i][p] for i, p in rows])
        low = np.concatenate([self.low[i][p] for i, p in rows])
        self.got = torch.full((len(proj), self.sh.heads, self.sh.vdim), float("nan"), dtype=TORCH[self.dt], device="cuda")
        return (dev(proj, self.dt), self.ld, dev(self.pad(low)), *self.weights, self.state, self.got)

    def check(self, rows, what):
        close(host(self.got), np.concatenate([self.out[i][p] for i, p in rows]), self.dt, what)

    def spans(self, cuts, kernel):
        """cuts: (sequence, slot, first, last) of one batch"""
        meta, row = [], 0
        for i, slot, a, b in cuts:
            meta.append((row, b - a, a, slot))
            row += b - a
        rows = [(i, slice(a, b)) for i, _, a, b in cuts]
        sp, n = ints(meta), len(meta)
        if kernel == "scan":
            call("lsh_lm_gla_scan_" + self.dt, *self.args(rows), sp, n, self.sh)
        else:
            from lightseq_amd import lib
            ws = torch.full((lib.load().lsh_lm_gla_chunked_workspace(row, n, ctypes.addressof(self.sh)),), float("nan"),
                            device="cuda")
            call("lsh_lm_gla_chunked_" + self.dt, *self.args(rows), ws, sp, n, max(m[1] for m in meta), row, self.sh)
        self.check(rows, "%s %s" % (kernel, cuts))

    def step(self, rows):
        """rows: (sequence, slot, position), one token each"""
        at = [(i, slice(p, p + 1)) for i, _, p in rows]
        call("lsh_lm_gla_step_" + self.dt, *self.args(at), ints([s for _, s, _ in rows]), ints([p for _, _, p in rows]),
             len(rows), self.sh)
        self.check(at, "step %s" % rows)

    def kernels(self):
        from lightseq_amd import lib
        ok = lib.load().lsh_lm_gla_chunked_supported(ctypes.addressof(self.sh), self.ld)
        return ("scan", "chunked") if ok else ("scan",)


CASES = [
    # H, D, VD, rank, tau
    (4, 32, 32, 16, 16.0), (3, 64, 48, 8, 1.0), (2, 80, 16, 20, 4.0), (1, 16, 144, 5, 8.0), (2, 128, 128, 16, 16.0),
    (2, 192, 256, 33, 16.0), (1, 256, 64, 16, 2.0), (3, 21, 19, 3, 16.0), (2, 40, 130, 16, 1.0), (1, 66, 250, 16, 5.0),
    (2, 200, 40, 16, 3.0), (1, 130, 30, 7, 16.0),
]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("case", range(len(CASES)))
def test_gated_linear_attention(dt, case):
    H, D, VD, rank, tau = CASES[case]
    g = Gla(dt, H, D, VD, rank, tau, [131, 64, 7, 200], case)
    if "chunked" not in g.kernels():
        with pytest.raises(Exception, match="multiples of 16"):
            g.device(5)
            g.spans([(0, 0, 0, 4)], "chunked")
    assert ("chunked" in g.kernels()) == (D % 16 == 0 and VD % 16 == 0)
    for kernel in g.kernels():
        g.device(5)
        # whole sequences of unequal length in one batch
        g.spans([(0, 3, 0, 131), (1, 0, 0, 64), (2, 4, 0, 7), (3, 1, 0, 200)], kernel)
        for i, slot in ((0, 3), (1, 0), (2, 4), (3, 1)):
            close(host(g.state[slot]), g.S[i], "f32", "state")
        assert torch.isnan(g.state[2]).all()  # nobody's slot
        # portions, down to one and two tokens, on slots used before
        for a, b in ((0, 2), (2, 3), (3, 66), (66, 130), (130, 131)):
            g.spans([(3, 3, a, b), (0, 1, a, b)], kernel)
        close(host(g.state[1]), g.S[0], "f32", "state")
    # prompt, then decoding; a sequence decoded from its first token beside it
    g.device(5)
    g.spans([(0, 2, 0, 70)], g.kernels()[-1])
    for t in range(40):
        g.step([(0, 2, 70 + t), (1, 4, t)])
    g.step([(2, 2, 0), (0, 0, 0)])  # slot 2 again, by another sequence
    g.step([(2, 2, 1)])


@pytest.mark.parametrize("kernel", ["scan", "chunked"])
@pytest.mark.parametrize("decay", [-60.0, 14.0])
def test_extreme_decays(kernel, decay):
    """Channels that forget everything at once (where quotients of decays would overflow), and channels
    that forget nothing over many chunks."""
    g = Gla("f32", 2, 64, 32, 16, 1.0, [400], 3, decay=decay)
    g.bias[::3] = np.float32(-decay)  # the other kind beside them
    n, sh = 400, g.sh
    cols = lambda at, w: g.proj[0][:, at:at + 2 * w].reshape(n, 2, w)  # noqa: E731
    la = O.log_decay(g.low[0], np.eye(16), g.a2, g.bias, 1.0).reshape(n, 2, 64)
    o, S = O.linear_attention(cols(sh.q_col, 64) / 8, cols(sh.k_col, 64), cols(sh.v_col, 32), la)
    g.out[0] = O.rms_norm(o, g.norm, 1e-5) * O.silu(cols(sh.g_col, 32))
    g.S[0] = S.transpose(0, 2, 1)
    assert np.exp(la).min() < 1e-4 and np.exp(la).max() > 0.999
    g.device(1)
    g.spans([(0, 0, 0, 400)], kernel)
    close(host(g.state[0]), g.S[0], "f32", "state")


@pytest.mark.parametrize("kernel", ["scan", "chunked"])
def test_one_far_key_is_remembered(kernel):
    """Every key but the first is zero and nothing decays: each output is the first value, scaled."""
    g = Gla("f32", 1, 32, 16, 16, 16.0, [300], 5)
    g.bias[:] = 80.0
    g.a2[:] = 0
    k, v = g.sh.k_col, g.sh.v_col
    g.proj[0][1:, k:k + 32] = 0
    q = g.proj[0][:, g.sh.q_col:g.sh.q_col + 32]
    share = (q @ g.proj[0][0, k:k + 32]) / np.sqrt(32)
    o = share[:, None, None] * g.proj[0][0, v:v + 16]
    g.out[0] = O.rms_norm(o, g.norm, 1e-5) * O.silu(g.proj[0][:, g.sh.g_col:g.sh.g_col + 16])[:, None]
    g.device(1)
    g.spans([(0, 0, 0, 130)], kernel)
    g.spans([(0, 0, 130, 299)], kernel)
    g.step([(0, 0, 299)])


def test_bad_shapes_are_refused():
    from lightseq_amd.lib import LSHError
    x, i = torch.zeros(64, device="cuda"), ints([0, 1, 0, 0])
    for sh, match in ((GlaShape(1, 300, 8, 16, 0, 0, 0, 0, 1.0, 0.0), "256"), (GlaShape(1, 8, 8, 5, 0, 0, 0, 0, 1.0, 0.0), "bad shape")):
        with pytest.raises(LSHError, match=match):
            call("lsh_lm_gla_scan_f32", x, 8, x, x, x, x, x, x, i, 1, sh)
    with pytest.raises(LSHError, match="activation"):
        call("lsh_lm_gemm_gated_f32", x, 8, x, x, 8, 1, 8, 8, 7)
