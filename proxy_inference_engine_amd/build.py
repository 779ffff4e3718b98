"""Builds the native libraries (hand-written HIP for gfx950) in-tree with hipcc.

    python -m proxy_inference_engine_amd.build [--force]

libpie_base.so: error plumbing, page pool, the 16-bit GEMM, the layer-stack models -- everything a layer-stack model needs, and all that
build_base() compiles (the trace runner in a fresh checkout).  libpie_hip.so: the Llama decoder, the quantised formats, the vision tower,
sampling; it links the base library.  hipcc cross-compiles without a GPU, so this runs in the build container; the libraries are git-ignored
and travel to the GPU box with the repo snapshot.
"""
from __future__ import annotations

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

PKG = Path(__file__).resolve().parent
CSRC = PKG / "csrc"
LIB_DIR = PKG / "lib"
LIB = LIB_DIR / "libpie_hip.so"
BASE_LIB = LIB_DIR / "libpie_base.so"
BASE_SOURCES = ["base.hip", "w16_gemm.hip", "w16_grouped.hip", "rows_gemm.hip", "latent_attn.hip", "window_attn.hip", "page_attn.hip", "delta_rule.hip", "gated_delta.hip", "time_mix.hip", "mlstm.hip", "mingru.hip", "head_out.hip", "row_update.hip", "stream_update.hip", "layer_stack.hip", "page_pool.cpp"]
SOURCES = ["w4_gemv.hip", "ops.hip", "decoder.hip", "prefill.hip", "vision.hip", "w4m_gemm.hip", "tp_comm.hip", "sampler.hip", "paged_i8.hip"]
# packed-fp32-ops off: hipcc otherwise forms v_pk_{add,mul,fma}_f32 from ordinary float code, and some of their forms are not reliable here
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off", "-fno-fast-math",
         "-Wall", "-Wno-unused-function", "-D__HIP_PLATFORM_AMD__"]
HIP_FLAGS = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if cand and (os.path.isabs(cand) and os.path.exists(cand) or not os.path.isabs(cand)):
            return cand
    raise RuntimeError("hipcc not found")


def _headers() -> list[Path]:
    return list(CSRC.glob("*.hpp")) + [PKG.parent / "include" / "pie_hip.h"]


def source_hash() -> str:
    """sha256 over the sources the library is built from: pie_version() carries its first 12 digits, and the counter files under
    profiles/ name the build they were measured on (bench.py refuses a stale one)."""
    import hashlib
    h = hashlib.sha256()
    for f in sorted(list(CSRC.glob("*.hip")) + list(CSRC.glob("*.hpp")) + list(CSRC.glob("*.cpp")) + [PKG.parent / "include" / "pie_hip.h"]):
        h.update(f.name.encode())
        h.update(f.read_bytes())
    return h.hexdigest()[:12]


def _make(lib: Path, sources: list[str], extra_link: list[str], deps: list[Path], force: bool, verbose: bool) -> Path:
    """Compiles what changed of `sources` and links `lib` when anything did."""
    stamps = [f.stat().st_mtime for f in [CSRC / src for src in sources] + _headers() + deps]
    if not force and lib.exists() and lib.stat().st_mtime >= max(stamps):
        return lib
    LIB_DIR.mkdir(exist_ok=True)
    obj_dir = LIB_DIR / "obj"
    obj_dir.mkdir(exist_ok=True)
    hipcc = _hipcc()
    newest_header = max(h.stat().st_mtime for h in _headers())

    def compile_one(src: str) -> bool:
        obj = obj_dir / (src + ".o")
        stamp = max(newest_header, (CSRC / src).stat().st_mtime)
        if src == "base.hip":  # carries the hash of all sources
            stamp = max([stamp] + [f.stat().st_mtime for f in list(CSRC.glob("*.hip")) + list(CSRC.glob("*.cpp"))])
        if not force and obj.exists() and obj.stat().st_mtime > stamp:
            return False
        extra = [f'-DPIE_BUILD_HASH="{source_hash()}"'] if src == "base.hip" else []
        cmd = [hipcc, *FLAGS, *(HIP_FLAGS if src.endswith(".hip") else []), *extra, "-c", str(CSRC / src), "-o", str(obj)]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed for {src}:\n{r.stderr[-6000:]}")
        if verbose and r.stderr.strip():
            print("\n".join(ln for ln in r.stderr.splitlines() if "packed-fp32-ops" not in ln), file=sys.stderr)
        return True

    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        changed = any(list(ex.map(compile_one, sources)))
    objs = [obj_dir / (s + ".o") for s in sources]
    if changed or not lib.exists() or any(o.stat().st_mtime > lib.stat().st_mtime for o in objs + deps):
        cmd = [hipcc, "--offload-arch=gfx950", "-shared", "-fPIC", f"-Wl,-soname,{lib.name}", "-o", str(lib), *map(str, objs), *extra_link]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"link failed:\n{r.stderr[-4000:]}")
    return lib


def build_base(force: bool = False, verbose: bool = False) -> Path:
    return _make(BASE_LIB, BASE_SOURCES, [], [], force, verbose)


def build(force: bool = False, verbose: bool = False) -> Path:
    base = build_base(force, verbose)
    return _make(LIB, SOURCES, [f"-L{LIB_DIR}", "-lpie_base", "-Wl,-rpath,$ORIGIN", "-ldl"], [base], force, verbose)


if __name__ == "__main__":
    print(build(force="--force" in sys.argv, verbose=True))
