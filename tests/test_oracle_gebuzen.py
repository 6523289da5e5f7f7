"""The plain Gebuzen decoder against properties and closed forms of its mechanisms, and the loader's
refusals (no GPU)."""
import json

import numpy as np
import pytest

from oracle import gebuzen as O
from tests import gebuzen_models as M
from tests.sudevik_models import row_errors

CONFIGS = {"aligned": M.ALIGNED, "odd": M.ODD, "large_heads": M.LARGE_HEADS, "plain": M.PLAIN}


def test_chunk_edges():
    m = {"size": 4}
    assert [j for j in range(12) if O.sees(9, j, m)] == [8, 9]
    assert [j for j in range(12) if O.sees(8, j, m)] == [8]
    assert [j for j in range(12) if O.sees(7, j, m)] == [4, 5, 6, 7]
    assert [j for j in range(4) if O.sees(2, j, None)] == [0, 1, 2]


def test_sink_takes_its_share():
    assert np.allclose(O.sink_softmax(np.array([0.0, 0.0]), 0.0), [1 / 3, 1 / 3])
    assert np.allclose(O.sink_softmax(np.array([1.0]), 1.0 + np.log(3.0)), [0.25])
    assert np.allclose(O.sink_softmax(np.array([5.0]), 1000.0), [0.0])
    assert np.allclose(O.sink_softmax(np.array([1000.0, 999.0]), -5.0).sum(), 1.0)


def test_grouped_heads_and_keys_as_values():
    r = np.random.default_rng(0)
    q, k = r.normal(size=(3, 4, 5)), r.normal(size=(3, 2, 5))
    o = O.attend(q, k, k, 0.7, {"size": 2}, np.full(4, -1e9))
    for h in range(4):  # position 2 opens a chunk: it sees itself only
        assert np.allclose(o[2, h], k[2, h // 2])
        s = np.exp(0.7 * k[:2, h // 2] @ q[1, h])
        assert np.allclose(o[1, h], s @ k[:2, h // 2] / s.sum())


def test_linear_attention_decays_key_channels():
    q = np.array([[[1.0, 10.0]], [[1.0, 10.0]]])
    k = np.array([[[1.0, 1.0]], [[0.0, 0.0]]])
    v = np.array([[[2.0, 3.0, 4.0]], [[9.0, 9.0, 9.0]]])
    la = np.log(np.array([[[0.1, 0.1]], [[0.5, 0.25]]]))
    o, S = O.linear_attention(q, k, v, la)
    assert np.allclose(o[0, 0], 11 * v[0, 0])  # the token's own write is not decayed
    assert np.allclose(o[1, 0], (0.5 + 2.5) * v[0, 0])
    assert np.allclose(S[0], [[1.0, 1.5, 2.0], [0.5, 0.75, 1.0]])
    o2, S2 = O.linear_attention(q[1:], k[1:], v[1:], la[1:], state=np.array([np.outer([1, 1], v[0, 0])]))
    assert np.allclose(o2[0], o[1]) and np.allclose(S2, S)


def test_decay_is_a_root_of_the_sigmoid():
    h, eye = np.array([[0.3, -2.0]]), np.eye(2)
    la = O.log_decay(h, eye, 2 * eye, np.array([0.1, 0.2]), 4.0)
    assert np.allclose(np.exp(la) ** 4, 1 / (1 + np.exp(-np.array([[0.7, -3.8]]))))


def test_layer_runs():
    assert O.layer_runs(M.ALIGNED) == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (1, 2), (2, 2), (3, None)]
    assert O.layer_runs(M.ODD) == [(0, 0), (1, 0), (2, 0), (0, 1), (1, 1), (2, 1)]
    assert O.layer_runs(M.PLAIN) == [(0, None), (1, None)]


@pytest.mark.parametrize("name", list(CONFIGS))
def test_causality(name):
    cfg = CONFIGS[name]
    t = O.widen(M.random_tensors(cfg, 1, M.RANKS[name]))
    r = np.random.default_rng(2)
    a = r.integers(0, cfg["vocab"], 30)
    b = a.copy()
    b[20:] = (b[20:] + 1) % cfg["vocab"]
    x, y = O.forward(cfg, t, a), O.forward(cfg, t, b)
    assert np.array_equal(x[:20], y[:20]) and not np.allclose(x[20:], y[20:])


@pytest.mark.parametrize("what", ["chunk", "sink", "state", "pass", "step", "tau", "scale", "residual_mult"])
def test_the_test_weights_show_every_mechanism(what):
    """A mistake planted in a mechanism of the oracle moves the logits well beyond the tolerances that
    the library is held to."""
    cfg = json.loads(json.dumps(M.ALIGNED))
    t = M.random_tensors(cfg, 11)
    toks = np.random.default_rng(5).integers(0, cfg["vocab"], 80)
    want = O.forward(cfg, t, toks)
    for l in cfg["layers"]:
        left, right = l["mixer"]["left"], l["mixer"]["right"]
        if what == "chunk":
            left["mask"]["size"] += 1
        elif what == "tau":
            right["tau"] *= 1.1
        elif what == "scale":
            left["scale"] *= 1.05
    if what == "sink":
        t = {k: v * 0 if k.endswith("sink") else v for k, v in t.items()}
    elif what == "state":
        t = {k: v - 1 if k.endswith("a2.b") else v for k, v in t.items()}
    elif what == "pass":
        cfg["loop"]["times"] = 2
    elif what == "step":
        t["loop.step"] = t["loop.step"][::-1]
    elif what == "residual_mult":
        cfg["residual_mult"] *= 1.05
    e = row_errors(O.forward(cfg, t, toks), want)
    assert e[-20:].max() > 0.01, e


# -- what the library refuses before it touches a GPU ---------------------------------------------
def changed(path, value):
    cfg = json.loads(json.dumps(M.ALIGNED))
    at = cfg
    for p in path[:-1]:
        at = at[p]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return cfg


@pytest.mark.parametrize("path,value,match", [
    (["layers", 0, "type"], "delta", "unknown layer type 'delta'"),
    (["layers", 0, "mixer", "left", "heads"], 3, "multiple of kv_heads"),
    (["layers", 0, "mixer", "left", "vdim"], 32, "vdim must be dim"),
    (["layers", 0, "mixer", "left", "scale"], None, "'scale' is missing"),
    (["layers", 0, "mixer", "left", "mask", "size"], 0, "'size' must be a positive integer"),
    (["layers", 2, "mixer", "right", "tau"], 0, "'tau' must be positive"),
    (["layers", 2, "mixer", "right"], None, "'right' is missing"),
    (["layers", 1, "mlp", "kind"], "moe", "unknown mlp kind 'moe'"),
    (["layers", 1, "mlp", "ff"], None, "'ff' is missing"),
    (["loop", "stop"], 5, "run of layers"),
    (["loop", "start"], 3, "run of layers"),
    (["loop", "times"], 0, "'times' must be a positive integer"),
    (["residual_mult"], None, "'residual_mult' is missing"),
    (["logit_scale"], None, "'logit_scale' is missing"),
    (["layers"], [], "no layers"),
])
def test_bad_configurations_are_refused(tmp_path, path, value, match):
    from lightseq_amd.inference import DecoderModel
    from lightseq_amd.lib import LSHError
    (tmp_path / "config.json").write_text(json.dumps(changed(path, value)))
    with pytest.raises(LSHError, match=match):
        DecoderModel(tmp_path)
