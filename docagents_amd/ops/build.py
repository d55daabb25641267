"""Build the gfx950 kernel libraries with hipcc — no hipify, no torch headers.

Every ``csrc/*.hip`` file is compiled to an object with ``hipcc --offload-arch=gfx950`` (in
parallel) and the objects of a part are linked into that part's shared library next to this file:

    gemm     _da_gemm.so      matrix products
    token    _da_token.so     norms, embeddings, pooling, RoPE, samplers
    hybrid   _da_hybrid.so    recurrent mixers, paged attention, 32-bit residual stream, fp32 products
    kernels  _da_kernels.so   everything else (attention, vector search, collectives, runtime)

A process loads (and, in a checkout without built libraries, compiles) only the parts it calls. The
libraries export plain ``extern "C"`` launchers (``da_*``) that take raw device pointers and a
``hipStream_t``; Python binds them with ctypes (``docagents_amd.ops.kernels``), so launches go onto
PyTorch's current HIP stream and are capturable in HIP graphs.

The libraries link against ``libamdhip64.so.7`` by SONAME; when PyTorch is imported first, the
dynamic loader resolves it to the HIP runtime PyTorch already loaded (one runtime per process).

Usage: ``python -m docagents_amd.ops.build [--force] [--debug]``
"""
from __future__ import annotations

import argparse
import concurrent.futures as cf
import hashlib
import os
import shutil
import subprocess
import sys
from pathlib import Path

HERE = Path(__file__).resolve().parent
CSRC = HERE / "csrc"
ARCH = os.environ.get("DA_OFFLOAD_ARCH", "gfx950")

_PART_SOURCES = {
    "gemm": ("gemm.hip", "gemm256.hip", "gemm4w.hip", "gemm8p.hip", "gemm_dk.hip"),
    "token": ("norm.hip", "rope_sample.hip"),
    "hybrid": ("delta.hip", "gemm_any.hip", "latent_attn.hip", "paged_attn.hip", "recurrent.hip", "stream_norm.hip"),
}
PARTS = (*_PART_SOURCES, "kernels")


def lib_path(part: str, debug: bool = False) -> Path:
    """The shared library of a part (debug: -O1 -g -DDA_DEBUG, device asserts on)."""
    return HERE / f"_da_{part}{'_debug' if debug else ''}.so"


def _stamp(part: str, debug: bool) -> Path:
    return HERE / f"_da_{part}{'_debug' if debug else ''}.fingerprint"


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", shutil.which("hipcc")):
        if cand and Path(cand).exists():
            return cand
    raise RuntimeError("hipcc not found (need ROCm >= 7.0)")


def _sources(part: str | None = None) -> list[Path]:
    if part in _PART_SOURCES:
        return [CSRC / n for n in _PART_SOURCES[part]]
    every = sorted(CSRC.glob("*.hip"))
    if part is None:
        return every
    named = {n for names in _PART_SOURCES.values() for n in names}
    return [p for p in every if p.name not in named]


def _fingerprint(part: str, debug: bool) -> str:
    h = hashlib.sha256()
    for p in sorted([*_sources(part), *CSRC.glob("*.h")]):
        h.update(p.name.encode())
        h.update(p.read_bytes())
    h.update(f"{_flags(debug)}".encode())
    return h.hexdigest()


def _flags(debug: bool) -> list[str]:
    # packed fp32 instructions off: some of their forms give wrong results on this hardware
    f = [f"--offload-arch={ARCH}", "-std=c++17", "-fPIC", "-mcode-object-version=5",
         "-Wno-unused-result", "-ffp-contract=fast", "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
    f += ["-O1", "-g", "-DDA_DEBUG=1"] if debug else ["-O3"]
    return f


LAST_BUILD: dict = {}


def source_hashes() -> dict:
    """sha256 (first 16 hex) of every kernel source: what a build compiled."""
    return {p.name: hashlib.sha256(p.read_bytes()).hexdigest()[:16] for p in sorted(CSRC.glob("*"))}


def _fresh(part: str, debug: bool) -> bool:
    lib, stamp = lib_path(part, debug), _stamp(part, debug)
    return lib.exists() and stamp.exists() and stamp.read_text() == _fingerprint(part, debug)


def build(force: bool = False, debug: bool = False, verbose: bool = False, parts=PARTS) -> dict[str, Path]:
    """Compile the stale ones of ``parts`` (all of them with ``force``) and return their libraries.
    ``LAST_BUILD`` records what happened: mode "compiled" (hipcc ran, with the wall time) or "reused"
    (fingerprint match)."""
    import time
    libs = {p: lib_path(p, debug) for p in parts}
    LAST_BUILD.clear()
    LAST_BUILD.update({"libs": [str(p) for p in libs.values()], "arch": ARCH, "debug": debug, "mode": "reused"})
    if not force and all(_fresh(p, debug) for p in parts):
        return libs
    # N ranks of one job import the package at once: one builds, the others wait and reuse it
    import fcntl
    with open(HERE / "_da_kernels.lock", "w") as lk:
        fcntl.flock(lk, fcntl.LOCK_EX)
        todo = [p for p in parts if force or not _fresh(p, debug)]
        if todo:
            t0 = time.perf_counter()
            _build_locked(todo, debug, verbose)
            LAST_BUILD.update({"mode": "compiled", "parts": todo, "compile_s": round(time.perf_counter() - t0, 1),
                               "sources": source_hashes()})
    return libs


def _build_locked(parts, debug: bool, verbose: bool) -> None:
    hipcc = _hipcc()
    objdir = HERE / ("_build_debug" if debug else "_build")
    objdir.mkdir(exist_ok=True)
    flags = _flags(debug)
    stamps = {p: _fingerprint(p, debug) for p in parts}

    def compile_one(src: Path) -> Path:
        obj = objdir / (src.stem + ".o")
        cmd = [hipcc, *flags, "-c", str(src), "-o", str(obj)]
        if verbose:
            print(" ".join(cmd), file=sys.stderr)
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed for {src.name}:\n{r.stderr}")
        return obj

    srcs = [s for p in parts for s in _sources(p)]
    workers = min(len(srcs), int(os.environ.get("MAX_JOBS", "8")), 16)
    with cf.ThreadPoolExecutor(max_workers=max(1, workers)) as ex:
        objs = dict(zip(srcs, ex.map(compile_one, srcs)))
    for p in parts:
        lib = lib_path(p, debug)
        tmp = lib.with_suffix(f".so.tmp{os.getpid()}")
        cmd = [hipcc, f"--offload-arch={ARCH}", "-shared", "-fPIC", *(str(objs[s]) for s in _sources(p)), "-o", str(tmp)]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"link failed:\n{r.stderr}")
        # a kernel whose launch stub the host pass dropped (e.g. a template-dependent array extent in a
        # builtin argument) links fine and fails only at dlopen on the GPU box: catch it here
        nm = shutil.which("nm")
        if nm:
            u = subprocess.run([nm, "-D", "--undefined-only", str(tmp)], capture_output=True, text=True).stdout
            stubs = [ln.split()[-1] for ln in u.splitlines() if "__device_stub__" in ln]
            if stubs:
                tmp.unlink(missing_ok=True)
                raise RuntimeError(f"undefined kernel launch stubs: {stubs[:4]}")
        os.replace(tmp, lib)
        _stamp(p, debug).write_text(stamps[p])


def main() -> None:
    ap = argparse.ArgumentParser()
    ap.add_argument("--force", action="store_true")
    ap.add_argument("--debug", action="store_true")
    ap.add_argument("-v", "--verbose", action="store_true")
    a = ap.parse_args()
    for p in build(force=a.force, debug=a.debug, verbose=a.verbose).values():
        print(p)


if __name__ == "__main__":
    main()
