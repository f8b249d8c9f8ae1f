"""Builds the HIP libraries (gfx950) from socket_amd/csrc with hipcc.

Run as `python -m socket_amd.build`; `__graft_entry__.build()` calls `build()`.
Objects are compiled in parallel, one translation unit per kernel family, and
linked into two libraries next to this file: libsocket_core.so (what every model
family uses: decode-step helpers, dense attention, chunked and latent attention,
gated recurrences) and libsocket_hip.so (hashing, scoring, selection and block-sparse
attention of the SOCKET path), which depends on it.  `build_core()` makes the first
alone.
"""
from __future__ import annotations

import os
import shutil
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB_PATH = os.path.join(HERE, "libsocket_hip.so")
CORE_PATH = os.path.join(HERE, "libsocket_core.so")
CORE_SOURCES = ["common.hip", "attend.hip", "decode_ops.hip", "rows.hip", "chunk_attend.hip", "latent.hip",
                "recurrence.hip"]
SOURCES = ["score.hip", "collide.hip", "topk.hip", "hash.hip", "softhash.hip", "block_sparse.hip"]
ARCH = "gfx950"
# Packed-FP32 VALU ops are switched off for every device translation unit.
FLAGS = [
    f"--offload-arch={ARCH}", "-O3", "-fPIC", "-std=c++17",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-Wno-unused-command-line-argument",
]


# Per-file additions.  block_sparse.hip: keep MFMA accumulators in ordinary
# registers (its softmax reads and rescales them every tile; the default form
# parks them in the accumulator file and moves them back and forth).
FILE_FLAGS = {
    "block_sparse.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],
    "attend.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],     # the MFMA dense flash-decode, for the same reason
    "chunk_attend.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],
    "latent.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],
    "recurrence.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],
}


def _hipcc() -> str:
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(exe):
        raise RuntimeError("hipcc not found; the HIP libraries cannot be built")
    return exe


def _run(cmd):
    p = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    if p.returncode != 0:
        raise RuntimeError("command failed: %s\n%s" % (" ".join(cmd), p.stdout))
    lines = [ln for ln in p.stdout.splitlines() if "not a recognized feature" not in ln]
    return "\n".join(lines)


def _stale(src_path: str, obj: str) -> bool:
    """True if the object is older than its source or any header."""
    if not os.path.exists(obj):
        return True
    t = os.path.getmtime(obj)
    deps = [src_path, os.path.join(HERE, "..", "include", "socket_hip.h")]
    deps += [os.path.join(CSRC, f) for f in os.listdir(CSRC) if f.endswith(".h")]
    return any(os.path.getmtime(d) > t for d in deps)


def _compile(sources, verbose: bool, extra_flags, only_changed: bool):
    hipcc = _hipcc()
    objdir = os.path.join(HERE, "build")
    os.makedirs(objdir, exist_ok=True)

    def compile_one(src):
        obj = os.path.join(objdir, src.replace(".hip", ".o"))
        if only_changed and not _stale(os.path.join(CSRC, src), obj):
            return obj
        out = _run([hipcc, *FLAGS, *FILE_FLAGS.get(src, []), *extra_flags, "-c", os.path.join(CSRC, src), "-o", obj])
        if verbose and out.strip():
            print(out)
        return obj

    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        return list(ex.map(compile_one, sources))


def _link(objs, path: str, *more) -> None:
    tmp = "%s.%d.tmp" % (path, os.getpid())
    _run([_hipcc(), f"--offload-arch={ARCH}", "-shared", "-fPIC", *objs, *more,
          "-Wl,-soname," + os.path.basename(path), "-o", tmp])
    os.replace(tmp, path)


def build_core(verbose: bool = False, extra_flags=(), only_changed: bool = False) -> str:
    """Compile and link libsocket_core.so alone."""
    _link(_compile(CORE_SOURCES, verbose, extra_flags, only_changed), CORE_PATH)
    return CORE_PATH


def build(verbose: bool = False, extra_flags=(), only_changed: bool = False) -> str:
    """Compile every source (or, with only_changed, those newer than their
    object) and link both libraries."""
    n = len(CORE_SOURCES)
    objs = _compile(CORE_SOURCES + SOURCES, verbose, extra_flags, only_changed)
    _link(objs[:n], CORE_PATH)
    _link(objs[n:], LIB_PATH, CORE_PATH, "-Wl,-rpath,$ORIGIN")
    return LIB_PATH


if __name__ == "__main__":
    run = build_core if "--core" in sys.argv else build
    print(run(verbose="-v" in sys.argv, only_changed="--changed" in sys.argv))
