"""Compile the HIP sources in csrc/ (gfx950) in-tree with hipcc: one library per element type.

    libmlora_hip.so    fp16: the Llama / LoRA hot path
    libmlora_bf16.so   bfloat16: the linear and row kernels and those of the latent-attention decoders
    libmlora_f32.so    fp32: the same decoders in IEEE fp32

Usage: python build.py [--force]
"""
from __future__ import annotations

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
SOURCES = ["api.hip", "gather_mm.hip", "gather_mm_batch.hip", "gemv.hip", "gemm.hip", "rowops.hip", "attention.hip", "decode_step.hip"]
DECODER_SOURCES = ["stream_ops.hip", "latent_attention.hip", "time_mix.hip", "moe.hip"]
LIBS = {   # element type -> (library, sources, suffix of the objects, extra flags)
    "float16": (os.path.join(HERE, "libmlora_hip.so"), SOURCES, "", []),
    "bfloat16": (os.path.join(HERE, "libmlora_bf16.so"), ["api.hip", "gemv.hip", "gemm.hip", "rowops.hip", *DECODER_SOURCES], "_bf16",
                 ["-DMLORA_ELT_BF16"]),
    "float32": (os.path.join(HERE, "libmlora_f32.so"), ["api.hip", "rowops.hip", "linear_f32.hip", *DECODER_SOURCES], "_f32", ["-DMLORA_ELT_F32"]),
}
LIB = LIBS["float16"][0]
HEADERS = [os.path.join(CSRC, h) for h in ("common.h", "lora_device.h", "gather_mm_batch.h", "moe.h")] + \
          [os.path.join(HERE, "..", "include", h) for h in ("mlora.h", "mlora_decoder.h")]
FLAGS = ["--offload-arch=gfx950", "-O3", "-fPIC", "-std=c++17", "-mllvm", "-amdgpu-kernarg-preload-count=16",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if cand and (os.path.isabs(cand) and os.path.exists(cand) or not os.path.isabs(cand)):
            return cand
    return "hipcc"


def _run(cmd):
    p = subprocess.run(cmd, capture_output=True, text=True)
    # the host pass prints a harmless "not a recognized feature" line for the packed-fp32 switch
    err = "\n".join(l for l in p.stderr.splitlines() if "packed-fp32-ops" not in l)
    if p.returncode != 0:
        raise RuntimeError(f"{' '.join(cmd)}\n{err}")
    if err.strip():
        sys.stderr.write(err + "\n")


def build(force: bool = True, jobs: int = 0, dtypes=tuple(LIBS)) -> str:
    """Compile every source of the libraries of `dtypes` to an object and link them; returns the path of the last one.
    jobs: compiler processes at once (0: MAX_JOBS, else 6)."""
    jobs = jobs or int(os.environ.get("MAX_JOBS") or 6)
    hdr_m = max(os.path.getmtime(h) for h in HEADERS)
    todo, links = [], []
    for dt in dtypes:
        lib, sources, suffix, extra = LIBS[dt]
        objs, stale = [], force or not os.path.exists(lib)
        for src in sources:
            s = os.path.join(CSRC, src)
            o = os.path.join(CSRC, src.replace(".hip", suffix + ".o"))
            objs.append(o)
            if force or not os.path.exists(o) or os.path.getmtime(o) < max(os.path.getmtime(s), hdr_m):
                todo.append([_hipcc(), *FLAGS, *extra, "-c", s, "-o", o])
                stale = True
        if stale or any(os.path.getmtime(o) > os.path.getmtime(lib) for o in objs):
            links.append([_hipcc(), "--offload-arch=gfx950", "-shared", "-fPIC", *objs, "-o", lib])
    with ThreadPoolExecutor(max_workers=jobs) as ex:
        list(ex.map(_run, todo))
    for cmd in links:
        _run(cmd)
    return LIBS[dtypes[-1]][0]


def ensure(dtype: str) -> str:
    """Build the library of one element type if it is not there (a fresh checkout); returns its path."""
    lib = LIBS[dtype][0]
    return lib if os.path.exists(lib) else build(force=False, dtypes=(dtype,))


if __name__ == "__main__":
    print(build(force="--force" in sys.argv))
