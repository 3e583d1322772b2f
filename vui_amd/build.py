"""Builds libvui_amd.so (gfx950) in-tree with hipcc.  `python -m vui_amd.build`."""
from __future__ import annotations

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB = os.path.join(HERE, "libvui_amd.so")
# the token language models alone: their kernels, the sampler, the graph helpers
LM_LIB = os.path.join(HERE, "libvui_lm.so")
LM_SOURCES = ["runtime.hip", "misc.hip", "sample_wide.hip", "lm_gemm.hip", "latent.hip", "scan.hip", "rows.hip", "sigattn.hip",
              "gla.hip", "moe.hip", "sandwich.hip", "lm.hip"]
SOURCES = ["gemv.hip", "gemm16.hip", "attn.hip", "misc.hip", "frame.hip", "rqbatch.hip", "bbatch.hip", "prefill.hip", "codec.hip", "api.hip",
           "runtime.hip", "sample_wide.hip", "lm_gemm.hip", "latent.hip", "scan.hip", "rows.hip", "sigattn.hip", "gla.hip", "moe.hip",
           "sandwich.hip", "lm.hip"]
FLAGS = [
    "-O3", "--offload-arch=gfx950", "-fPIC", "-std=c++17", "-Wall", "-Wno-unused-function",
    # packed-fp32 instructions are kept out of every code object of this library
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
]


def _hipcc() -> str:
    for p in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if p and (os.path.sep not in p or os.path.exists(p)):
            return p
    return "hipcc"


def _build(lib: str, sources: "list[str]", verbose: bool) -> str:
    hipcc = _hipcc()
    extra = os.environ.get("VUI_EXTRA_HIPCC_FLAGS", "").split()
    objdir = os.path.join(CSRC, "build")
    os.makedirs(objdir, exist_ok=True)

    def one(src: str) -> str:
        obj = os.path.join(objdir, src.replace(".hip", ".o"))
        cmd = [hipcc, *FLAGS, *extra, "-c", os.path.join(CSRC, src), "-o", obj]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed on {src}:\n{r.stdout}\n{r.stderr}")
        if verbose and r.stderr.strip():
            lines = [l for l in r.stderr.splitlines() if "packed-fp32-ops" not in l and l.strip()]
            if lines:
                print("\n".join(lines), file=sys.stderr)
        return obj

    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        objs = list(ex.map(one, sources))
    tmp = lib + ".tmp"
    cmd = [hipcc, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", tmp, *objs]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"link failed:\n{r.stdout}\n{r.stderr}")
    os.replace(tmp, lib)  # a library is there whole or not at all
    if verbose:
        print(f"built {lib}")
    return lib


def build(verbose: bool = True) -> str:
    """Compiles every translation unit and links the shared library.  Always recompiles."""
    return _build(LIB, SOURCES, verbose)


def build_lm(verbose: bool = True) -> str:
    """The part of the library that serves the token language models.  Always recompiles."""
    return _build(LM_LIB, LM_SOURCES, verbose)


if __name__ == "__main__":
    build()
