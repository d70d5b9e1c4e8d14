"""Build libmi355llama.so (gfx950) in-tree with hipcc.

No torch linkage: the library is a plain C-ABI shared object (include/mi355_llama.h) that only needs the
HIP runtime, which `_native.py` makes sure is the instance PyTorch already loaded.
"""
from __future__ import annotations

import os
import shutil
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

PKG = Path(__file__).resolve().parent
CSRC = PKG / "csrc"
LIB = PKG / "libmi355llama.so"
CORE_LIB = PKG / "libmi355core.so"
OBJ_DIR = PKG / "csrc" / "_obj"
# what a layered hybrid model runs on; linked alone into CORE_LIB where only such a model is served
CORE_SOURCES = ["generic.hip", "gemv.hip", "gemm.hip", "sample.hip", "graph.hip", "window_attention.hip", "recurrent.hip",
                "recurrent_chunks.hip", "latent_attention.hip", "experts.hip", "join.hip", "hybrid.hip"]
SOURCES = CORE_SOURCES + ["int8.hip", "int8_gemm.hip", "attention.hip", "engine.hip", "gptq.hip", "fused_step.hip", "fused_step_ring.hip",
                          "fused_step_wide.hip", "tp_comm.hip", "flash_prefill.hip"]
ARCH = "gfx950"
# hipcc -O3 turns ordinary float code into packed-f32 instructions, some forms of which have given wrong results on these
# machines; the host pass says it does not know the feature, which is harmless
NO_PACKED_F32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", shutil.which("hipcc")):
        if cand and Path(cand).exists():
            return cand
    raise RuntimeError("hipcc not found (looked at $HIPCC, /opt/rocm/bin/hipcc, PATH)")


def _stale(target: Path, deps) -> bool:
    if not target.exists():
        return True
    t = target.stat().st_mtime
    return any(Path(d).stat().st_mtime > t for d in deps)


def build_core(force: bool = False, verbose: bool = True) -> Path:
    """The part of the library that a layered hybrid model needs (a fresh checkout that serves one compiles no more)."""
    return build(force, verbose, CORE_SOURCES, CORE_LIB)


def build(force: bool = False, verbose: bool = True, sources=None, lib: Path = LIB) -> Path:
    sources = SOURCES if sources is None else sources
    hipcc = _hipcc()
    OBJ_DIR.mkdir(exist_ok=True)
    headers = [CSRC / "common.h", CSRC / "fused_step_common.h", CSRC / "gemm_fuse.h", CSRC / "recurrent.h", CSRC / "product.h", PKG.parent / "include" / "mi355_llama.h"]
    flags = [f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function", *NO_PACKED_F32]

    def compile_one(name: str):
        src = CSRC / name
        obj = OBJ_DIR / (name + ".o")
        if force or _stale(obj, [src, *headers]):
            cmd = [hipcc, *flags, "-c", str(src), "-o", str(obj)]
            if verbose:
                print(" ".join(cmd), file=sys.stderr)
            r = subprocess.run(cmd, capture_output=True, text=True)
            if r.returncode != 0:
                raise RuntimeError(f"hipcc failed on {name}:\n{r.stdout}\n{r.stderr}")
            if verbose and r.stderr.strip():
                print(r.stderr, file=sys.stderr)
        return obj

    compiled = []

    def compile_tracked(name: str):
        obj = OBJ_DIR / (name + ".o")
        before = obj.stat().st_mtime if obj.exists() else None
        out = compile_one(name)
        if before is None or out.stat().st_mtime != before:
            compiled.append(name)
        return out

    with ThreadPoolExecutor(max_workers=min(len(sources), os.cpu_count() or 4)) as ex:
        objs = list(ex.map(compile_tracked, sources))
    relink = force or _stale(lib, objs)
    if verbose:  # say what this call did: an up-to-date tree compiles nothing, and the caller should see that
        print(f"[build] {len(sources)} sources for {ARCH}: compiled {sorted(compiled) if compiled else 'none (objects up to date)'}; "
              f"{'linking' if relink else 'library up to date:'} {lib}", file=sys.stderr)
    if relink:
        cmd = [hipcc, f"--offload-arch={ARCH}", "-shared", "-fPIC", "-o", str(lib), *map(str, objs)]
        if verbose:
            print(" ".join(cmd), file=sys.stderr)
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"link failed:\n{r.stdout}\n{r.stderr}")
    return lib


if __name__ == "__main__":
    print(build(force="--force" in sys.argv))
