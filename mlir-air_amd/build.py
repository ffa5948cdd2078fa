"""Build the HIP libraries (gfx950) in-tree with hipcc.

    python mlir-air_amd/build.py [-j JOBS] [--only NAME ...]

Output: mlir-air_amd/lib/libw4a16_hip.so (int4 weights) and mlir-air_amd/lib/libdense_lm_hip.so (dense weights).  Each
stands alone, so a program that serves one kind of model builds only what it needs (`ensure`).  Cross-compiles without a
GPU.
"""

import argparse
import concurrent.futures
import contextlib
import fcntl
import os
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
OBJ_DIR = os.path.join(HERE, "build")
LIB_DIR = os.path.join(HERE, "lib")
LIBRARIES = {
    "w4a16": ["capi.hip", "dequant.hip", "stream.hip", "gemv_ws.hip", "gemm_ws.hip", "gemm_wsk.hip", "gemm.hip", "attention.hip", "q4nx.hip", "lm_head.hip", "prefill_block.hip", "prefill_attention.hip"],
    "dense_lm": ["dense_capi.hip", "dense_gemv.hip", "dense_gemm.hip", "rows.hip", "moe.hip", "latent_attention.hip", "latent_prefill.hip",
                 "head_attention.hip", "linear_attention.hip", "linear_chunks.hip", "mixer_steps.hip"],
}
SOURCES = [s for sources in LIBRARIES.values() for s in sources]


def lib_path(name):
    return os.path.join(LIB_DIR, f"lib{name}_hip.so")


LIB_PATH = lib_path("w4a16")

HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
FLAGS = [
    *os.environ.get("W4A16_EXTRA", "").split(),
    "--offload-arch=gfx950",
    "-O3",
    "-std=c++17",
    "-fPIC",
    "-Wall",
    "-Wno-unused-function",
    # packed fp32 VALU ops are kept out of every kernel
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    # the first kernel arguments arrive in SGPRs with the wave instead of through scalar loads at its start
    # (decode GEMV 6.09 -> 5.88 us); only kernels with plain scalar / pointer arguments gain
    "-mllvm", "-amdgpu-kernarg-preload-count=16",
]


# Per-file flags.  The prompt-pass attentions take maxima over MFMA results: without the promise that they are not
# NaN the compiler canonicalises every one of them first (one more VALU instruction per score).
FILE_FLAGS = {"prefill_attention.hip": ["-fno-honor-nans"], "latent_prefill.hip": ["-fno-honor-nans"]}


def _compile(src, extra):
    obj = os.path.join(OBJ_DIR, os.path.splitext(src)[0] + ".o")
    cmd = [HIPCC, *FLAGS, *FILE_FLAGS.get(src, []), *extra, "-c", os.path.join(CSRC, src), "-o", obj]
    res = subprocess.run(cmd, capture_output=True, text=True)
    out = "\n".join(
        line for line in (res.stdout + res.stderr).splitlines()
        if "packed-fp32-ops" not in line and "unrecognized feature" not in line
    )
    if res.returncode != 0:
        raise RuntimeError(f"hipcc failed for {src}:\n{out}")
    return obj, out


def build(jobs=4, extra=(), verbose=False, only=None):
    """Compile and link the libraries named in `only` (default: all); returns the path of the last one."""
    names = list(only or LIBRARIES)
    os.makedirs(OBJ_DIR, exist_ok=True)
    os.makedirs(LIB_DIR, exist_ok=True)
    sources = [s for name in names for s in LIBRARIES[name]]
    with concurrent.futures.ThreadPoolExecutor(max_workers=jobs) as pool:
        results = dict(zip(sources, pool.map(lambda s: _compile(s, list(extra)), sources)))
    for _, out in results.values():
        if out.strip() and verbose:
            print(out)
    for name in names:
        objs = [results[s][0] for s in LIBRARIES[name]]
        tmp = f"{lib_path(name)}.{os.getpid()}"   # renamed when whole: nobody loads half a library
        subprocess.check_call([HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", tmp, *objs])
        os.replace(tmp, lib_path(name))
    return lib_path(names[-1])


@contextlib.contextmanager
def _lock():
    os.makedirs(OBJ_DIR, exist_ok=True)
    with open(os.path.join(OBJ_DIR, ".lock"), "w") as f:
        fcntl.flock(f, fcntl.LOCK_EX)
        yield


def ensure(name, jobs=8):
    """The library `name`, built first if there is none (one builder at a time)."""
    if not os.path.exists(lib_path(name)):
        with _lock():
            if not os.path.exists(lib_path(name)):
                build(jobs, only=[name])
    return lib_path(name)


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("-j", type=int, default=4)
    ap.add_argument("-v", action="store_true")
    ap.add_argument("--only", nargs="*", choices=list(LIBRARIES), help="build these libraries only")
    ap.add_argument("--save-temps", action="store_true", help="keep ISA (.s) files under build/")
    a = ap.parse_args()
    extra = ["-save-temps=obj"] if a.save_temps else []
    print(build(a.j, extra, a.v or True, a.only))
