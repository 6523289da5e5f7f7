"""Builds ``liblightseq_hip.so`` (every HIP kernel + the C ABI) for gfx950 with hipcc.

``python -m lightseq_amd.build`` compiles each translation unit of ``csrc/`` to an
object file (in parallel) and links them into ``lightseq_amd/lib/``.  The GPU is not
needed: hipcc cross-compiles.  ``build_decoder_library`` builds the part that the
floating-point decoder models need, ``liblightseq_decoder.so``: the same model C ABI
without the int8 kernels and models.
"""
import concurrent.futures
import fcntl
import os
import shutil
import subprocess
import sys

_HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(_HERE, "csrc")
OBJ_DIR = os.path.join(CSRC, "_obj")
LIB_DIR = os.path.join(_HERE, "lib")
LIB_PATH = os.path.join(LIB_DIR, "liblightseq_hip.so")
DECODER_LIB_PATH = os.path.join(LIB_DIR, "liblightseq_decoder.so")

# sources of liblightseq_decoder.so
DECODER_SOURCES = [
    "core.hip", "gemm_float.hip", "lm_norm_kernels.hip", "lm_attn_kernels.hip", "delta_kernels.hip",
    "gla_kernels.hip", "moe_kernels.hip", "lm_sample_kernels.hip", "lm_capi.hip",
    "model/model_capi.cpp", "model/model_dir.cpp", "model/decoder_lm.cpp", "model/sudevik.cpp",
    "model/sudevik_config.cpp", "model/sudevik_decoder.cpp", "model/sudevik_weight.cpp",
    "model/gebuzen.cpp", "model/gebuzen_config.cpp", "model/gebuzen_decoder.cpp",
    "model/gebuzen_weight.cpp",
]

ARCH = "gfx950"
# -packed-fp32-ops off: hipcc must not form v_pk_{add,mul,fma}_f32 from float code.
HIPCC_FLAGS = [
    "-O3", "-std=c++17", "-fPIC", "--offload-arch=" + ARCH, "-Wall", "-Wno-unused-function",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
]


def _hipcc():
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(exe):
        raise RuntimeError("hipcc not found")
    return exe


def sources():
    out = []
    for root, _dirs, files in os.walk(CSRC):
        if os.path.basename(root) == "_obj":
            continue
        for f in sorted(files):
            if f.endswith(".hip") or f.endswith(".cpp"):
                out.append(os.path.join(root, f))
    return sorted(out)


def _compile_one(src):
    rel = os.path.relpath(src, CSRC).replace(os.sep, "_")
    obj = os.path.join(OBJ_DIR, os.path.splitext(rel)[0] + ".o")
    cmd = [_hipcc()] + HIPCC_FLAGS + ["-x", "hip", "-c", src, "-o", obj]
    p = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    # the host pass does not know the device-only target feature; drop that one line
    log = "\n".join(l for l in p.stdout.splitlines() if "packed-fp32-ops" not in l)
    if p.returncode != 0:
        raise RuntimeError("hipcc failed for %s:\n%s" % (src, log))
    return obj, log


def build_library(verbose=False, jobs=None):
    """Compile everything and link the shared library; returns its path."""
    return _build(sources(), LIB_PATH, verbose, jobs)


def build_decoder_library(verbose=False, jobs=None):
    """The library of the floating-point decoder models only; returns its path."""
    return _build([os.path.join(CSRC, s) for s in DECODER_SOURCES], DECODER_LIB_PATH, verbose, jobs)


def ensure_decoder_library():
    """Path of a built library that has the decoder models, building the smaller one if there is
    none.  Safe when several processes call it at once."""
    if os.path.exists(LIB_PATH):
        return LIB_PATH
    os.makedirs(LIB_DIR, exist_ok=True)
    with open(os.path.join(LIB_DIR, ".build_lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if os.path.exists(DECODER_LIB_PATH):
            return DECODER_LIB_PATH
        return build_decoder_library()


def _build(srcs, lib_path, verbose, jobs):
    os.makedirs(OBJ_DIR, exist_ok=True)
    os.makedirs(LIB_DIR, exist_ok=True)
    jobs = jobs or min(8, len(srcs))
    objs = []
    with concurrent.futures.ThreadPoolExecutor(max_workers=jobs) as ex:
        for obj, log in ex.map(_compile_one, srcs):
            objs.append(obj)
            if verbose and log.strip():
                print(log)
    cmd = [_hipcc(), "-shared", "-fPIC", "--offload-arch=" + ARCH, "-o", lib_path + ".part"] + objs
    p = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    if p.returncode != 0:
        raise RuntimeError("link failed:\n" + p.stdout)
    os.replace(lib_path + ".part", lib_path)
    return lib_path


if __name__ == "__main__":
    path = build_library(verbose=True)
    print("built", path)
    sys.exit(0)
