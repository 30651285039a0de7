"""Compiling the HIP sources for gfx950 and loading the result.

Libraries are built with ``hipcc`` into ``csrc/_build`` inside the package (or, when that is not
writable, into a per-user folder under the temporary directory) and loaded with ``ctypes``.  A
library is rebuilt when its sources or flags change.  The core library holds every kernel whose
sizes are run-time arguments; the matrix-core attention kernels keep their accumulators in
registers and address pages with constant arithmetic; they are therefore compiled once per (head size,
page size), on first use of that pair.

There is no fallback: if ``hipcc`` is missing or a source does not compile, loading raises.
"""

from __future__ import annotations

import ctypes
import hashlib
import os
import shutil
import subprocess
import sys
import tempfile
import threading
import time
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

CSRC = Path(__file__).resolve().parent.parent / "csrc"
ARCH = "gfx950"
FLAGS = ["-O3", "-std=c++17", "-fPIC", "-shared", f"--offload-arch={ARCH}",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops", "-Wno-unused-command-line-argument"]

CORE_SOURCES = ["elementwise.hip", "gemm_generic.hip", "attn_generic.hip", "sampling.hip", "gemm_bf16.hip", "gemm_wide.hip", "graph.hip", "streams.hip", "delta.hip", "latent.hip", "memory.hip", "moe.hip", "retention.hip", "mamba.hip"]
ATTN_SOURCES = ["attn_mfma.hip"]
WIDE_SOURCES = ["attn_wide.hip"]

_loaded: dict[str, ctypes.CDLL] = {}


_build_dir_found: Path | None = None
_build_dir_lock = threading.Lock()


def _build_dir() -> Path:
    """Where libraries are built: beside the sources, or a per-user temporary folder if that cannot be written.  Found
    once per process (several compilers run at a time, and all of them must land in the same place)."""
    global _build_dir_found
    with _build_dir_lock:
        if _build_dir_found is None:
            d = CSRC / "_build"
            try:
                d.mkdir(exist_ok=True)
                probe = d / f".w{os.getpid()}"
                probe.write_text("")
                probe.unlink()
            except OSError:
                d = Path(tempfile.gettempdir()) / f"nanospec_amd_build_{os.getuid()}"
                d.mkdir(parents=True, exist_ok=True)
            _build_dir_found = d
        return _build_dir_found


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), shutil.which("hipcc"), "/opt/rocm/bin/hipcc"):
        if cand and Path(cand).exists():
            return cand
    raise RuntimeError("nanospec_amd needs hipcc (ROCm) to build its kernels; none was found")


def _digest(sources: list[str], defines: list[str]) -> str:
    h = hashlib.sha256()
    for name in sorted(set(sources) | {h.name for h in CSRC.glob("*.h")}):
        h.update(name.encode())
        h.update((CSRC / name).read_bytes())
    h.update(" ".join(FLAGS + defines).encode())
    return h.hexdigest()


def _say(msg: str) -> None:
    print(f"[nanospec_amd] {msg}", file=sys.stderr, flush=True)


def _run_hipcc(name: str, t0: float, args: list[str]) -> None:
    """One hipcc run; a line every 15 seconds while it works; raises with its output if it fails."""
    proc = subprocess.Popen([_hipcc(), *args], stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    while True:
        try:
            log, _ = proc.communicate(timeout=15)
            break
        except subprocess.TimeoutExpired:
            _say(f"  still compiling lib{name}.so, {time.time() - t0:.0f} s")
    if proc.returncode != 0:
        Path(args[-1]).unlink(missing_ok=True)
        log = "\n".join(l for l in log.splitlines() if "packed-fp32-ops" not in l)
        raise RuntimeError(f"hipcc failed for lib{name}.so:\n{log}")


def compile_library(name: str, sources: list[str], defines: list[str] = (), force: bool = False) -> Path:
    """Build ``lib<name>.so`` if it is missing or stale (or ``force``); return its path."""
    defines = list(defines)
    out_dir = _build_dir()
    lib = out_dir / f"lib{name}.so"
    stamp = out_dir / f"lib{name}.sha256"
    digest = _digest(sources, defines)
    if not force and lib.exists() and stamp.exists() and stamp.read_text().strip() == digest:
        return lib
    tmp = out_dir / f"lib{name}.{os.getpid()}.tmp.so"
    _say(f"compiling lib{name}.so for {ARCH} ({', '.join(sources)}) ...")
    t0 = time.time()
    if len(sources) == 1:
        _run_hipcc(name, t0, [*FLAGS, *defines, str(CSRC / sources[0]), "-o", str(tmp)])
    else:
        # one object a source, several compilers at a time, then one link
        objects = [out_dir / f"{name}.{Path(src).stem}.{os.getpid()}.tmp.o" for src in sources]
        flags = [f for f in FLAGS if f != "-shared"]
        try:
            with ThreadPoolExecutor(max_workers=max(1, min(8, os.cpu_count() or 1))) as pool:
                for done in [pool.submit(_run_hipcc, name, t0, [*flags, *defines, "-c", str(CSRC / src), "-o", str(obj)])
                             for src, obj in zip(sources, objects)]:
                    done.result()
            _run_hipcc(name, t0, [*FLAGS, *(str(o) for o in objects), "-o", str(tmp)])
        finally:
            for o in objects:
                o.unlink(missing_ok=True)
    os.replace(tmp, lib)
    stamp.write_text(digest)
    _say(f"built lib{name}.so in {time.time() - t0:.0f} s")
    return lib


def load_library(name: str, sources: list[str], defines: list[str] = ()) -> ctypes.CDLL:
    if name not in _loaded:
        path = compile_library(name, sources, defines)
        try:
            _loaded[name] = ctypes.CDLL(str(path))
        except OSError as e:
            raise RuntimeError(f"nanospec_amd could not load its kernel library {path}: {e}") from e
    return _loaded[name]


def core() -> ctypes.CDLL:
    return load_library("ns_core", CORE_SOURCES)


def attn_name(head_dim: int, page_size: int) -> str:
    return f"ns_attn_hd{head_dim}_p{page_size}"


def _attn_defines(head_dim: int, page_size: int) -> list[str]:
    return [f"-DNS_HEAD_DIM={head_dim}", f"-DNS_PAGE_SIZE={page_size}"]


def attn(head_dim: int, page_size: int) -> ctypes.CDLL:
    """The matrix-core attention kernels for one head size and one page size."""
    return load_library(attn_name(head_dim, page_size), ATTN_SOURCES, _attn_defines(head_dim, page_size))


def wide_name(head_dim: int, value_dim: int, page_size: int) -> str:
    return f"ns_wide_hd{head_dim}_v{value_dim}_p{page_size}"


def _wide_defines(head_dim: int, value_dim: int, page_size: int) -> list[str]:
    return [f"-DNS_HEAD_DIM={head_dim}", f"-DNS_VALUE_DIM={value_dim}", f"-DNS_PAGE_SIZE={page_size}"]


def attn_wide(head_dim: int, value_dim: int, page_size: int) -> ctypes.CDLL:
    """The matrix-core attention kernel for keys and values of two sizes (and wide heads), one library per (key size, value
    size, page size), compiled on first use."""
    return load_library(wide_name(head_dim, value_dim, page_size), WIDE_SOURCES, _wide_defines(head_dim, value_dim, page_size))


def build_all(attn_variants=((16, 4), (32, 8), (64, 16), (128, 16)), force: bool = True, jobs: int | None = None, wide_variants=()) -> None:
    """Compile the core library, the attention library of each given (head size, page size) and the two-size attention
    library of each given (key size, value size, page size), ``jobs`` compilers at a time (by default one per processor, at
    most eight)."""
    work = [("ns_core", CORE_SOURCES, [])] + [(attn_name(hd, page), ATTN_SOURCES, _attn_defines(hd, page)) for hd, page in attn_variants]
    work += [(wide_name(hd, vd, page), WIDE_SOURCES, _wide_defines(hd, vd, page)) for hd, vd, page in wide_variants]
    jobs = jobs or max(1, min(8, os.cpu_count() or 1))
    with ThreadPoolExecutor(max_workers=jobs) as pool:
        for done in [pool.submit(compile_library, name, sources, defines, force) for name, sources, defines in work]:
            done.result()
