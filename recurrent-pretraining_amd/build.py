"""Builds libraven_hip.so (gfx950) from csrc/*.hip with hipcc.  Run on the CPU container; the
built library travels to the GPU box with the tree."""

import os
import shutil
import subprocess
import sys

PKG_DIR = os.path.dirname(os.path.abspath(__file__))
ROOT = os.path.dirname(PKG_DIR)
CSRC = os.path.join(PKG_DIR, "csrc")
LIB_DIR = os.path.join(PKG_DIR, "lib")
LIB_PATH = os.path.join(LIB_DIR, "libraven_hip.so")
SOURCES = ["rmsnorm.hip", "gemm_skinny.hip", "gemm_splitk.hip", "gemm_tiled.hip", "gemv_decode.hip", "attention.hip", "attention_prefill.hip", "misc.hip", "exit_stats.hip", "compose.hip",
           "tuning.hip", "norm_conv.hip", "attention_capped.hip", "delta_rule.hip", "latent_attention.hip", "rglru.hip", "moe.hip",
           "compose_mixer.hip"]

HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",  # no packed-fp32 VALU forms
    "-Wall", "-Wno-unused-function",
]


def hipcc() -> str:
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(exe):
        raise RuntimeError("hipcc not found; libraven_hip.so cannot be built")
    return exe


def build_library(verbose: bool = True, sources=None, path: str = LIB_PATH) -> str:
    """Compiles `sources` (all by default) in parallel and links them into `path`."""
    os.makedirs(LIB_DIR, exist_ok=True)
    objs = []
    procs = []
    for src in (SOURCES if sources is None else sources):
        obj = os.path.join(LIB_DIR, src.replace(".hip", ".o"))
        cmd = [hipcc(), *HIPCC_FLAGS, "-I", os.path.join(ROOT, "include"), "-I", CSRC, "-c", os.path.join(CSRC, src), "-o", obj]
        procs.append((src, subprocess.Popen(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)))
        objs.append(obj)
    for src, p in procs:
        out, _ = p.communicate()
        out = "\n".join(l for l in out.splitlines() if "packed-fp32-ops" not in l)
        if p.returncode != 0:
            raise RuntimeError(f"hipcc failed on {src}:\n{out}")
        if verbose and out.strip():
            print(out, file=sys.stderr)
    part = f"{path}.{os.getpid()}.tmp"  # a process that loads the library meanwhile sees the old one or the new one
    link = [hipcc(), "--offload-arch=gfx950", "-shared", "-fPIC", "-Wl,-z,defs", "-o", part, *objs]
    r = subprocess.run(link, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"link failed:\n{r.stdout}")
    os.replace(part, path)
    return path


def ensure_library(name: str, sources=None) -> str:
    """Path of a built library that serves the model family `name`: the whole one when it has been built, else one of only the
    family's kernel sources, compiled now if need be."""
    if os.path.exists(LIB_PATH):
        return LIB_PATH
    if sources is None:
        return build_library(verbose=False)
    path = os.path.join(LIB_DIR, f"libraven_hip_{name}.so")
    return path if os.path.exists(path) else build_library(verbose=False, sources=sources, path=path)


if __name__ == "__main__":
    print(build_library())
