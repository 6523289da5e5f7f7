"""Whole Gebuzen models through the library's step and generation interfaces against the plain decoder:
prompts, decoding, portions, batches, used slots, generation."""
import json
import subprocess
import sys
import os

import numpy as np
import pytest
import torch

from oracle import gebuzen as O
from tests import gebuzen_models as G
from tests import sudevik_models as M

pytestmark = pytest.mark.gpu

CONFIGS = {"aligned": G.ALIGNED, "odd": G.ODD, "large_heads": G.LARGE_HEADS, "plain": G.PLAIN}
F32_TOL = 1e-4


class Case:
    def __init__(self, name, folder):
        self.cfg = CONFIGS[name]
        self.folder = str(folder)
        tensors = G.random_tensors(self.cfg, 11, G.RANKS[name])
        O.write_model(self.folder, self.cfg, tensors)
        self.t = O.widen(tensors)
        r = np.random.default_rng(5)
        self.tokens = {k: r.integers(0, self.cfg["vocab"], n).tolist()
                       for k, n in (("a", 150), ("b", 61), ("c", 1), ("d", 90))}
        self.want = {k: O.forward(self.cfg, self.t, v) for k, v in self.tokens.items()}

    def model(self, dtype="float32", **kw):
        from lightseq_amd.inference import DecoderModel
        return DecoderModel(self.folder, dtype, **dict(dict(max_batch_size=4, max_step=200), **kw))


@pytest.fixture(scope="module", params=list(CONFIGS))
def case(request, tmp_path_factory):
    return Case(request.param, tmp_path_factory.mktemp("gebuzen_" + request.param))


@pytest.fixture(scope="module")
def model(case):
    m = case.model()
    yield m
    m.close()


def check(got, want, tol=F32_TOL):
    e = M.row_errors(got, want)
    assert e.max() < tol, "row %d of %d: %.3g" % (int(e.argmax()), len(e), e.max())


def test_whole_prompts(case, model):
    f = M.Fed(model)
    for k, toks in case.tokens.items():
        check(f.feed({k: toks})[k], case.want[k])
        f.end(k)


def test_token_by_token_equals_the_prompt(case, model):
    f = M.Fed(model)
    got = np.concatenate([f.feed({"b": [t]})["b"] for t in case.tokens["b"]])
    check(got, case.want["b"])
    f.end("b")


@pytest.mark.parametrize("sizes", [(2,), (3, 1, 64), (70, 2, 1), (9, 17)])
def test_portions(case, model, sizes):
    f, got, at, i = M.Fed(model), [], 0, 0
    toks = case.tokens["a"]
    while at < len(toks):
        n = sizes[i % len(sizes)]
        got.append(f.feed({"a": toks[at:at + n]})["a"])
        at, i = at + n, i + 1
    check(np.concatenate(got), case.want["a"])
    f.end("a")


def test_unequal_batch_then_decoding_together(case, model):
    """Four requests start as one batch and are decoded together; the shorter ones end earlier."""
    f = M.Fed(model)
    start = {"a": 100, "b": 55, "c": 1, "d": 30}
    out = {k: [v] for k, v in f.feed({k: case.tokens[k][:n] for k, n in start.items()}).items()}
    f.end("c")
    live = {k: n for k, n in start.items() if k != "c"}
    while live:
        for k, v in f.feed({k: [case.tokens[k][n]] for k, n in live.items()}).items():
            out[k].append(v)
        live = {k: n + 1 for k, n in live.items()}
        for k in [k for k, n in live.items() if n == len(case.tokens[k])]:
            f.end(k)
            del live[k]
    for k in start:
        check(np.concatenate(out[k]), case.want[k])


def test_mixed_prompt_and_single_tokens(case, model):
    """A batch in which one sequence brings a prompt, others one token."""
    f = M.Fed(model)
    f.feed({"a": case.tokens["a"][:80]})
    got = f.feed({"b": case.tokens["b"][:40], "a": [case.tokens["a"][80]], "c": case.tokens["c"]})
    check(got["a"], case.want["a"][80:81])
    check(got["b"], case.want["b"][:40])
    check(got["c"], case.want["c"])
    check(f.feed({"a": [case.tokens["a"][81]], "b": [case.tokens["b"][40]]})["b"], case.want["b"][40:41])
    f.end("a", "b", "c")


def test_slots_are_reused_clean(case, model):
    """Long sequences leave their keys, states and convolution inputs behind; the next owner of the
    slot must not see them, neither from a prompt nor from a first decoding step."""
    f = M.Fed(model)
    for names in (["a", "d"], ["b", "c"], ["c", "b"], ["d", "a"]):
        got = f.feed({k: case.tokens[k][:40] for k in names})
        for k in names:
            check(got[k], case.want[k][:40])
        f.end(*names)
    first = f.feed({"d": case.tokens["d"][:1]})["d"]
    check(np.concatenate([first, f.feed({"d": case.tokens["d"][1:2]})["d"]]), case.want["d"][:2])
    f.end("d")


def test_wanted_rows_only(case, model):
    s = model.open_sequence()
    got = model.step([(s, case.tokens["d"])], [3, 88, 3])
    check(got, case.want["d"][[3, 88, 3]])
    assert model.step([(s, [1])]).shape == (0, case.cfg["vocab"])
    model.close_sequence(s)


def test_bfloat16(case):
    m = case.model("bfloat16")
    f = M.Fed(m)
    whole = {k: f.feed({k: v})[k] for k, v in case.tokens.items()}
    f.end(*whole)
    out = f.feed({k: v[:len(v) // 2 + 1] for k, v in case.tokens.items()})
    rows = {k: [v] for k, v in out.items()}
    live = [k for k in case.tokens if len(case.tokens[k]) > 1]
    n = {k: len(case.tokens[k]) // 2 + 1 for k in live}
    f.end("c")
    while live:
        got = f.feed({k: [case.tokens[k][n[k]]] for k in live})
        for k in list(live):
            rows[k].append(got[k])
            n[k] += 1
            if n[k] == len(case.tokens[k]):
                live.remove(k)
    for got in (whole, {k: np.concatenate(v) for k, v in rows.items()}):
        e = np.concatenate([M.row_errors(got[k], case.want[k]) for k in case.tokens])
        assert np.isfinite(e).all() and np.median(e) < 0.03 and e.max() < 0.15, (np.median(e), e.max())
    m.close()


def test_layer_taps(case, model):
    want = []
    toks = case.tokens["b"]
    O.forward(case.cfg, case.t, toks, want)
    buf = torch.zeros(len(toks), case.cfg["width"], device="cuda")
    for i, w in enumerate(want):
        s = model.open_sequence()
        model.set_tap(i, "dec.res_out", buf)
        model.set_tap_step(model.steps_run())
        model.step([(s, toks)])
        model.set_tap(i, "dec.res_out", None)
        model.close_sequence(s)
        assert np.abs(buf.cpu().numpy() - w).max() < 1e-4 * max(1.0, np.abs(w).max()), i


def test_long_decoding_passes_every_window(case):
    """One sequence decoded far beyond its prompt, the windows moving over decoded tokens."""
    toks = (case.tokens["a"] + case.tokens["d"])[:230]
    want = O.forward(case.cfg, case.t, toks)
    m = case.model(max_step=240, max_batch_size=1)
    f = M.Fed(m)
    got = [f.feed({"x": toks[:2]})["x"]] + [f.feed({"x": [t]})["x"] for t in toks[2:]]
    check(np.concatenate(got), want)
    m.close()


# -- generation -----------------------------------------------------------------------------------
def test_greedy_generation(case):
    prompts = [case.tokens["b"][:20], case.tokens["d"][:3], case.tokens["c"]]
    want = [O.greedy(case.cfg, case.t, p, 12) for p in prompts]
    m = case.model(extra_decode_length=12)
    assert m.generate(prompts) == want
    for p, w in zip(prompts, want):  # alone, on slots used before
        assert m.generate([p]) == [w]
    m.close()


def test_generation_as_graphs_is_the_same(case):
    m = case.model("bfloat16", extra_decode_length=30)
    prompts = [case.tokens["a"][:40], case.tokens["d"][:7]]
    eager = m.generate(prompts)
    m.graph_mode(True)
    for _ in range(3):
        assert m.generate(prompts) == eager
    captured, replayed = m.graph_stats()
    assert captured >= 1 and replayed >= 60 and m.graph_nodes() > 10
    # a longer prompt moves buffers: what was captured must not be used again
    longer = m.generate([case.tokens["a"][:120]] + prompts)
    m.graph_mode(False)
    assert m.generate([case.tokens["a"][:120]] + prompts) == longer
    m.close()


def test_generation_stops_at_eos(case):
    prompts = [case.tokens["b"][:20], case.tokens["d"][:3]]
    free = case.model(extra_decode_length=12)
    texts = free.generate(prompts)
    free.close()
    eos = texts[0][25]
    m = case.model(extra_decode_length=12, eos_id=eos, padding_id=-7)
    got = m.generate(prompts)
    for g, t, p in zip(got, texts, prompts):
        new = t[len(p):]
        assert g == p + (new[:new.index(eos) + 1] if eos in new else new)
    m.close()


def test_random_sampling_repeats_with_its_seed(case):
    m = case.model(topk=20, extra_decode_length=16)
    prompts = [case.tokens["b"][:20], case.tokens["d"][:3]]
    m.set_seed(3)
    a = m.generate(prompts)
    b = m.generate(prompts)
    m.set_seed(3)
    assert m.generate(prompts) == a and a != b
    m.close()
    m = case.model(topk=0, topp=1e-6, extra_decode_length=8)  # only the largest logit is left
    g = case.model(extra_decode_length=8)
    assert m.generate(prompts) == g.generate(prompts)
    m.close()
    g.close()


def test_limits_are_errors(case, model):
    from lightseq_amd.lib import LSHError
    slots = [model.open_sequence() for _ in range(4)]
    with pytest.raises(LSHError, match="no free sequence slot"):
        model.open_sequence()
    with pytest.raises(LSHError, match="longer than max_step"):
        model.step([(slots[0], [1] * 201)])
    with pytest.raises(LSHError, match="outside the vocabulary"):
        model.step([(slots[0], [case.cfg["vocab"]])])
    with pytest.raises(LSHError, match="twice"):
        model.step([(slots[0], [1]), (slots[0], [1])])
    with pytest.raises(LSHError, match="outside the step"):
        model.step([(slots[0], [1])], [1])
    for s in slots:
        model.close_sequence(s)
    with pytest.raises(LSHError, match="not an open sequence"):
        model.step([(slots[0], [1])])
    with pytest.raises(LSHError, match="no profiled encoder"):
        model.set_profiling(True)


def test_trace_and_generate_command_lines(case, tmp_path):
    """The two programs, as child processes."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = case.tokens["a"], case.tokens["b"]
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:9], "want": [0, 8]},
                                     {"id": "y", "tokens": b[:5], "want": [4]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[9:10], "want": []}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": a[10:11], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "z", "tokens": b[:3], "want": [2]}], "end": ["z"]}]
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", case.folder, "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "64"], text=True, capture_output=True, timeout=100,
                       input="".join(json.dumps(s) + "\n" for s in steps))
    assert p.returncode == 0, p.stderr
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == ["done %d" % i for i in range(4)]
    got = [np.fromfile(tmp_path / ("%d.f32" % i), "<f4").reshape(-1, case.cfg["vocab"]) for i in (0, 2, 3)]
    check(got[0], np.stack([case.want["a"][0], case.want["a"][8], case.want["b"][4]]))
    check(got[1], case.want["a"][10:11])
    check(got[2], case.want["b"][2:3])
    assert not (tmp_path / "1.f32").exists()
    p = subprocess.run([sys.executable, "-m", "lightseq_amd.generate", "--model", case.folder, "--dtype", "float32",
                        "--ids", " ".join(map(str, b[:6])), "--ids", "3", "--new", "5"], text=True, cwd=root,
                       capture_output=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert p.stdout.splitlines()[-2:] == [" ".join(map(str, O.greedy(case.cfg, case.t, x, 5))) for x in (b[:6], [3])]
