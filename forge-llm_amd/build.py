"""Compile libforge_hip.so for gfx950 with hipcc (in-tree; no GPU needed to build)."""
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
INCLUDE = os.path.join(os.path.dirname(HERE), "include")
BUILD = os.path.join(HERE, "build")
LIB = os.path.join(HERE, "libforge_hip.so")

SOURCES = ["format.hip", "elementwise.hip", "gemv.hip", "gemv_f32.hip", "gemv_kquant.hip", "kquant_prefill.hip", "gemm.hip", "attn_decode.hip", "attn_prefill.hip",
           "attn_exact.hip", "decode_persistent.hip", "api.hip", "model.hip", "llama.hip", "block_model.hip", "block_mixers.hip", "dense.hip",
           "attn_prompt.hip", "attn_latent.hip", "attn_grouped.hip", "linear_attn.hip", "checkpoint.cpp", "gguf.cpp", "sampling.cpp"]

# The trace replay program holds the dense networks only.
TRACE_RUN = os.path.join(BUILD, "trace_run")
TRACE_SOURCES = ["format.hip", "elementwise.hip", "model.hip", "block_model.hip", "block_mixers.hip", "dense.hip", "attn_prompt.hip", "attn_latent.hip", "attn_grouped.hip",
                 "linear_attn.hip", "checkpoint.cpp", "trace_run.cpp"]

# -packed-fp32-ops off: keep hipcc from forming packed FP32 instructions.
# -ffp-contract=off: the CPU path never fuses a*b+c; kernels say fmaf() where a fused op is meant.
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function", "-Wno-pass-failed", "-ffp-contract=off",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
         "-I", INCLUDE, "-I", CSRC]


def _hipcc():
    for c in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if c and (os.path.isabs(c) and os.path.exists(c) or not os.path.isabs(c)):
            return c
    return "hipcc"


def _compile(src):
    obj = os.path.join(BUILD, os.path.splitext(src)[0] + ".o")
    part = "%s.%d" % (obj, os.getpid())
    cmd = [_hipcc(), *FLAGS, "-c", os.path.join(CSRC, src), "-o", part]
    r = subprocess.run(cmd, capture_output=True, text=True)
    # the host pass warns that it does not know the packed-fp32 feature: harmless, filter it
    err = "\n".join(l for l in r.stderr.splitlines() if "packed-fp32-ops" not in l)
    if r.returncode != 0:
        raise RuntimeError(f"hipcc failed on {src}:\n{err}")
    if err.strip():
        sys.stderr.write(err + "\n")
    os.replace(part, obj)
    return obj


def _link(out, objs, *flags):
    part = "%s.%d" % (out, os.getpid())
    r = subprocess.run([_hipcc(), "--offload-arch=gfx950", *flags, "-o", part, *objs], capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError("link failed:\n" + r.stderr)
    os.replace(part, out)


def _compile_all(sources):
    os.makedirs(BUILD, exist_ok=True)
    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        return list(ex.map(_compile, sources))


def build(verbose=True):
    objs = _compile_all(SOURCES + ["trace_run.cpp"])
    _link(LIB, objs[:-1], "-shared", "-fPIC")
    by_name = dict(zip(SOURCES + ["trace_run.cpp"], objs))
    _link(TRACE_RUN, [by_name[s] for s in TRACE_SOURCES])
    if verbose:
        print(f"built {LIB}")
    return LIB


def _older(path, than):
    return not os.path.exists(path) or os.path.getmtime(path) < than


def build_trace_run():
    """The trace replay program, compiled if it is not there or older than its sources."""
    headers = [os.path.join(d, f) for d in (CSRC, INCLUDE) for f in os.listdir(d) if f.endswith(".h")] + [os.path.abspath(__file__)]
    newest_header = max(os.path.getmtime(h) for h in headers)
    newest = max([newest_header] + [os.path.getmtime(os.path.join(CSRC, s)) for s in TRACE_SOURCES])
    if _older(TRACE_RUN, newest):
        obj = lambda s: os.path.join(BUILD, os.path.splitext(s)[0] + ".o")
        stale = [s for s in TRACE_SOURCES if _older(obj(s), max(newest_header, os.path.getmtime(os.path.join(CSRC, s))))]
        if stale:
            _compile_all(stale)
        _link(TRACE_RUN, [obj(s) for s in TRACE_SOURCES])
    return TRACE_RUN


if __name__ == "__main__":
    build()
