"""Generates token ids with a model in a folder::

    python -m lightseq_amd.generate --model DIR --ids "5 17 3" --ids "8" --new 32

One line of ids per prompt (``--ids``, or lines of standard input) comes out, prompt first.
"""
import argparse
import sys


def main(argv=None):
    ap = argparse.ArgumentParser(prog="lightseq_amd.generate", description=__doc__.split("::")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--ids", action="append", default=[], help="a prompt; may be given several times")
    ap.add_argument("--new", type=int, default=32, help="tokens after the longest prompt")
    ap.add_argument("--topk", type=int, default=1, help="1: greedy; 0: use --topp")
    ap.add_argument("--topp", type=float, default=0.75)
    ap.add_argument("--eos", type=int, default=-1)
    ap.add_argument("--seed", type=int, default=0)
    a = ap.parse_args(argv)
    prompts = [[int(t) for t in p.split()] for p in (a.ids or sys.stdin) if p.strip()]
    if not prompts:
        ap.error("no prompt")
    from . import build, lib
    lib.load(build.ensure_decoder_library())
    from .inference import DecoderModel
    model = DecoderModel(a.model, a.dtype, max_batch_size=len(prompts),
                         max_step=max(map(len, prompts)) + a.new, topk=a.topk, topp=a.topp,
                         eos_id=a.eos, extra_decode_length=a.new)
    model.set_seed(a.seed)
    for row in model.generate(prompts):
        print(" ".join(map(str, row)), flush=True)
    model.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
