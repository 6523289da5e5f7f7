"""Replays a trace of given tokens through a model in a folder and writes logits.

Steps come on standard input, one JSON object a line::

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Every entry appends tokens to its sequence (a new id opens one); all entries of a step are one
batch.  ``want`` names the tokens whose logits go to ``<out>/<step>.f32`` as little-endian float32
``[wanted, vocab]``, ``end`` the sequences to close after the step.  ``done <step>`` is printed after
each step.  Nothing is sampled.
"""
import argparse
import json
import os
import sys


class Replay:
    """Feeds steps to a model; sequences are named by the trace's ids."""

    MIN_SLOTS = 64

    def __init__(self, model_dir, dtype, max_tokens):
        self.model_dir, self.dtype, self.max_tokens = model_dir, dtype, max(int(max_tokens), 1)
        self.model, self.slots, self.live = None, 0, {}

    def _model_for(self, sequences):
        if self.model is None or sequences > self.slots:
            if self.live:
                raise RuntimeError("more live sequences than places")
            if self.model is not None:
                self.model.close()
            from .inference import DecoderModel
            self.slots = max(sequences, min(self.max_tokens, self.MIN_SLOTS))
            self.model = DecoderModel(self.model_dir, self.dtype, max_batch_size=self.slots,
                                      max_step=self.max_tokens)
        return self.model

    def step(self, entries, end=()):
        """Logits of the wanted tokens, in the order of the entries (None if nothing is wanted)."""
        out = None
        if entries:
            new = sum(e["id"] not in self.live for e in entries)
            model = self._model_for(len(self.live) + new)
            batch, want, row = [], [], 0
            for e in entries:
                if e["id"] not in self.live:
                    self.live[e["id"]] = model.open_sequence()
                batch.append((self.live[e["id"]], e["tokens"]))
                want += [row + w for w in e.get("want", ())]
                row += len(e["tokens"])
            logits = model.step(batch, want)
            out = logits if want else None
        for i in end:
            self.model.close_sequence(self.live.pop(i))
        return out


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096,
                    help="most tokens that live sequences hold at any time")
    a = ap.parse_args(argv)
    from . import build, lib
    lib.load(build.ensure_decoder_library())
    replay = Replay(a.model, a.dtype, a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = replay.step(s["entries"], s.get("end", ()))
        if logits is not None:
            logits.astype("<f4").tofile(os.path.join(a.out, "%d.f32" % s["step"]))
        print("done %d" % s["step"], flush=True)
    return 0
