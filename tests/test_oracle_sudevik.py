"""The plain Sudevik decoder against properties and closed forms of its mechanisms, and the loader's
refusals (no GPU)."""
import json
import math

import numpy as np
import pytest

from oracle import sudevik as O
from tests import sudevik_models as M


def test_yarn_frequencies_keep_fast_pairs_and_stretch_slow_ones():
    rot = M.yarn(10000.0, 64, 4.0, 4096, 32.0, 1.0)
    plain, one = O.rope_frequencies({"base": 10000.0, "dims": 64})
    f, mag = O.rope_frequencies(rot)
    assert one == 1.0 and abs(mag - (0.1 * math.log(4.0) + 1)) < 1e-15
    turns = 4096 * plain / (2 * math.pi)
    assert np.allclose(f[turns > 40], plain[turns > 40])
    assert np.allclose(f[turns < 0.8], plain[turns < 0.8] / 4)
    assert np.all(f <= plain * (1 + 1e-12)) and np.all(f >= plain / 4 * (1 - 1e-12))


def test_rotation_preserves_length_and_depends_on_distance_only():
    rot = {"base": 100.0, "dims": 6}
    r = np.random.default_rng(0)
    q, k = r.normal(size=(1, 1, 10)), r.normal(size=(1, 1, 10))
    a = O.rotate(q, [7], rot)[0, 0] @ O.rotate(k, [3], rot)[0, 0]
    b = O.rotate(q, [24], rot)[0, 0] @ O.rotate(k, [20], rot)[0, 0]
    assert abs(a - b) < 1e-12
    assert np.array_equal(O.rotate(q, [5], rot)[..., 6:], q[..., 6:])
    # the pair (0, 1) at position 1 turns by one radian
    x = np.zeros((1, 1, 10))
    x[..., 0] = 1
    assert np.allclose(O.rotate(x, [1], rot)[0, 0, :2], [math.cos(1), math.sin(1)])


def test_window_edges_and_kept_tokens():
    m = {"size": 4, "keep_first": 2}
    assert [j for j in range(12) if O.sees(9, j, m)] == [0, 1, 6, 7, 8, 9]
    assert [j for j in range(12) if O.sees(1, j, m)] == [0, 1]


def test_sink_takes_its_share():
    assert np.allclose(O.sink_softmax(np.array([0.0, 0.0])), [1 / 3, 1 / 3])
    assert np.allclose(O.sink_softmax(np.array([-1000.0])), [0.0])
    assert np.allclose(O.sink_softmax(np.array([1000.0, 999.0])).sum(), 1.0)


def test_delta_rule_reads_its_own_write_and_overwrites():
    k = np.zeros((2, 1, 3))
    k[:, 0, 1] = 1
    v = np.array([[[2.0, 5.0]], [[7.0, 1.0]]])
    one = np.ones((2, 1))
    o, S = O.delta_rule(k, k, v, one, one)
    assert np.allclose(o[:, 0], v[:, 0])  # the value of a key is replaced, not added to
    o2, _ = O.delta_rule(k, k, v, 0.5 * one, 0 * one, state=np.ones((1, 3, 2)))
    assert np.allclose(o2[:, 0], [[0.5, 0.5], [0.25, 0.25]])


def test_short_conv_last_column_is_the_current_token():
    x = np.arange(1.0, 5.0)[:, None]
    assert np.allclose(O.short_conv(x, np.array([[0.0, 0.0, 1.0]]))[:, 0], [1, 2, 3, 4])
    assert np.allclose(O.short_conv(x, np.array([[1.0, 0.0, 0.0]]))[:, 0], [0, 0, 1, 2])


def test_route_prefers_the_lower_index_among_equals():
    chosen, w = O.route(np.array([1.0, 3.0, 3.0, 2.0]), 2)
    assert chosen == [1, 2] and np.allclose(w, 0.5)


@pytest.mark.parametrize("cfg", [M.ALIGNED, M.ODD], ids=["aligned", "odd"])
def test_causality(cfg):
    t = O.widen(M.random_tensors(cfg, 1))
    r = np.random.default_rng(2)
    a = r.integers(0, cfg["vocab"], 30)
    b = a.copy()
    b[20:] = (b[20:] + 1) % cfg["vocab"]
    x, y = O.forward(cfg, t, a), O.forward(cfg, t, b)
    assert np.array_equal(x[:20], y[:20]) and not np.allclose(x[20:], y[20:])


def test_safetensors_round_trip(tmp_path):
    t = {"a": np.arange(6, dtype=np.float32).reshape(2, 3), "b": np.array([0.1], np.float32)}
    O.write_model(tmp_path, M.ODD, t)
    cfg, back = O.load_model(tmp_path)
    assert cfg == M.ODD and np.array_equal(back["a"], t["a"])
    assert np.array_equal(back["b"], O.round_bf16(t["b"]))


# -- what the library refuses before it touches a GPU ---------------------------------------------
def refused(tmp_path, cfg, match):
    from lightseq_amd.inference import DecoderModel
    from lightseq_amd.lib import LSHError
    (tmp_path / "config.json").write_text(cfg if isinstance(cfg, str) else json.dumps(cfg))
    with pytest.raises(LSHError, match=match):
        DecoderModel(tmp_path)


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
    (["architecture"], "Other", "Model not supported: Other"),
    (["architecture"], None, "'architecture' is missing"),
    (["width"], 0, "'width' must be a positive integer"),
    (["width"], 1.5, "integer"),
    (["norm", "eps"], None, "'eps' is missing"),
    (["layers"], [], "no layers"),
    (["layers", 0, "type"], "linear", "unknown layer type 'linear'"),
    (["layers", 0, "mixer", "heads"], 3, "multiple of kv_heads"),
    (["layers", 1, "mixer", "rot", "dims"], 66, "rot.dims"),
    (["layers", 1, "mixer", "scale"], None, "'scale' is missing"),
    (["layers", 3, "mixer", "kv_from"], 0, "kv_from"),
    (["layers", 3, "mixer", "kv_from"], 3, "kv_from"),
    (["layers", 3, "mixer", "dim"], 96, "other head sizes"),
    (["layers", 0, "mlp", "kind"], "dense", "unknown mlp kind 'dense'"),
    (["layers", 0, "mlp", "router", "top"], 11, "more choices"),
])
def test_bad_configurations_are_refused(tmp_path, path, value, match):
    refused(tmp_path, changed(path, value), match)


@pytest.mark.parametrize("text", ["", "{", "[1,]", '{"a" 1}', '{"a": tru}', '"\\x"', "{} x"])
def test_bad_json_is_refused(tmp_path, text):
    refused(tmp_path, text, "json")


def test_missing_folder_is_refused(tmp_path):
    from lightseq_amd.inference import DecoderModel
    from lightseq_amd.lib import LSHError
    with pytest.raises(LSHError, match="not found"):
        DecoderModel(tmp_path / "nothing")
    with pytest.raises(TypeError, match="unknown option"):
        DecoderModel(tmp_path, beam=4)


def test_decoder_library_is_a_subset():
    """The smaller library lists existing sources and needs nothing of the int8 models."""
    import os
    import re
    from lightseq_amd import build
    for s in build.DECODER_SOURCES:
        text = open(os.path.join(build.CSRC, s)).read()
        assert not re.search(r'#include "(?:\.\./)?(?:quant_|gemm_tile|dec_|gpt_)', text), s
