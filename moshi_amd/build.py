"""Build the engine libraries (HIP, gfx950 only) in-tree with hipcc.

    python -m moshi_amd.build            # build what is older than its sources
    python -m moshi_amd.build --force
    python -m moshi_amd.build tlm        # one library only

    mi    libmoshi_mi.so    codec, Moshi LM, session batcher, duplex pipeline (include/moshi_mi.h)
    tlm   libmoshi_tlm.so   token language models (include/moshi_tlm.h)

The libraries have no torch dependency: they are plain C-ABI shared objects that PyTorch-ROCm tensors are handed to by raw
device pointer.
"""
from __future__ import annotations

import os
import subprocess
import sys
from pathlib import Path

PKG = Path(__file__).resolve().parent
CSRC = PKG / "csrc"
ROOT = PKG.parent
LIB = PKG / "libmoshi_mi.so"
LIBS = {
    "mi": (LIB, ["api_common.hip", "mimi_engine.hip", "lm_engine.hip", "batcher.hip", "duplex.hip"]),
    "tlm": (PKG / "libmoshi_tlm.so", ["api_common.hip", "tlm_engine.hip"]),
}
ARCH = "gfx950"
# no v_pk_{add,mul,fma}_f32: some operand forms of the packed fp32 instructions have returned stale elements on gfx950
NO_PACKED_FP32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if cand and (os.path.isabs(cand) and os.path.exists(cand) or not os.path.isabs(cand)):
            return cand
    raise RuntimeError("hipcc not found")


def needs_build(which: str) -> bool:
    lib, _ = LIBS[which]
    if not lib.exists():
        return True
    t = lib.stat().st_mtime
    deps = list(CSRC.glob("*.h")) + list(CSRC.glob("*.hip")) + list((ROOT / "include").glob("*.h"))
    return any(p.stat().st_mtime > t for p in deps)


def build(force: bool = False, verbose: bool = True, which=None) -> Path:
    """Build the named libraries (default: all of them); returns the last one's path.  Several ranks of one node may call this at
    once (one process per GPU): the compile runs under a file lock, and a rank that waited for it finds the libraries up to date."""
    import fcntl
    names = list(LIBS) if which is None else [which] if isinstance(which, str) else list(which)
    with open(PKG / ".build.lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        try:
            return _build_locked(names, force, verbose)
        finally:
            fcntl.flock(lock, fcntl.LOCK_UN)


def _build_locked(names, force: bool, verbose: bool) -> Path:
    todo = [n for n in names if force or needs_build(n)]
    jobs = []
    for src in dict.fromkeys(s for n in todo for s in LIBS[n][1]):
        obj = CSRC / (Path(src).stem + ".o")
        cmd = [_hipcc(), f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off", *NO_PACKED_FP32,
               "-Wno-unused-result", "-Wno-unused-value", f"-I{CSRC}", "-c", str(CSRC / src), "-o", str(obj)]
        if verbose:
            print(" ".join(cmd), flush=True)
        jobs.append((subprocess.Popen(cmd, stdout=sys.stderr), cmd))
    for p, cmd in jobs:
        if p.wait() != 0:
            raise RuntimeError("hipcc failed: " + " ".join(cmd))
    for n in todo:
        lib, srcs = LIBS[n]
        cmd = [_hipcc(), f"--offload-arch={ARCH}", "-shared", "-fPIC", "-o", str(lib)] + [str(CSRC / (Path(s).stem + ".o")) for s in srcs]
        if verbose:
            print(" ".join(cmd), flush=True)
        subprocess.check_call(cmd, stdout=sys.stderr)
    return LIBS[names[-1]][0]


if __name__ == "__main__":
    picked = [a for a in sys.argv[1:] if not a.startswith("-")]
    print(build(force="--force" in sys.argv, which=picked or None))
