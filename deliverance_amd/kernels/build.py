"""Compiling the HIP sources for gfx950 into shared libraries, and loading them.

Every source is a unit of its own, ``deliverance_amd/csrc/_build/libda_<source>.so``, compiled in-tree with plain
``hipcc``; when that folder cannot be written, a folder under the system's temporary directory is used.  ``load()``
hands out entry points by name and loads the unit that holds one when it is first asked for; a unit that is not built
(or older than its source or a header) is compiled then.  ``ensure(units)`` compiles what is missing of a set side by
side, so that a model's first call in a fresh checkout compiles what that model needs; ``build(force=True)`` always
compiles everything.  There is no fallback: without the libraries and without ``hipcc`` the engine refuses to run.
"""
from __future__ import annotations

import ctypes
import fcntl
import glob
import hashlib
import os
import re
import shutil
import subprocess
import sys
import tempfile
import time
from concurrent.futures import ThreadPoolExecutor
from typing import Dict, Iterable, List, Optional, Sequence

CSRC = os.path.normpath(os.path.join(os.path.dirname(os.path.abspath(__file__)), "..", "csrc"))
ARCH = "gfx950"
# Packed 32-bit float instructions are switched off for all device code.
HIPCC_FLAGS = ["-O3", "-std=c++17", "-fPIC", f"--offload-arch={ARCH}",
               "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
               "-Wno-unused-result", "-Wno-unknown-warning-option"]
# Per unit: kernels that read their matrix-core results back at once (softmax between two
# products) keep them in ordinary vector registers; the default puts them into accumulation
# registers and moves every value out and in again.
EXTRA_FLAGS = {"attn_prefill": ["-mllvm", "-amdgpu-mfma-vgpr-form"],
               "attn_prefill_rel": ["-mllvm", "-amdgpu-mfma-vgpr-form"],
               "attn_latent_mfma": ["-mllvm", "-amdgpu-mfma-vgpr-form"],
               "attn_window": ["-mllvm", "-amdgpu-mfma-vgpr-form"]}
# The unit that holds the error message every entry point may leave; every other unit needs it.
BASE_UNIT = "rowwise"
# Units whose functions a unit calls.
NEEDS = {"gemm_mfma": ("gemm_wide",),
         "run_step": ("dispatch", "gemm_mfma", "gemm_fused", "attn_decode", "attn_prefill")}
# Units that are another unit's source compiled with a definition in front, and entry points that are not found by
# reading their unit's own source.
INCLUDES = {"attn_decode_rel": "attn_decode", "attn_prefill_rel": "attn_prefill"}
_ELSEWHERE = {"da_attn_decode_rel": "attn_decode_rel", "da_attn_prefill_rel": "attn_prefill_rel",
              "da_attn_prefill_rel_max_dist": "attn_prefill_rel", "da_gemm_wide_choice": "gemm_wide"}

_lib = None


class KernelLibraryError(RuntimeError):
    pass


def units() -> List[str]:
    return sorted(os.path.basename(p)[:-4] for p in glob.glob(os.path.join(CSRC, "*.hip")))


def _source(unit: str) -> str:
    return os.path.join(CSRC, unit + ".hip")


_entry_points: Optional[Dict[str, str]] = None


def entry_points() -> Dict[str, str]:
    """Entry point -> unit, read off the sources."""
    global _entry_points
    if _entry_points is None:
        found = {}
        for unit in units():
            with open(_source(unit)) as f:
                for name in re.findall(r'^extern "C" [\w *]*?\b(da_\w+)\s*\(', f.read(), re.M):
                    found[name] = unit
        found.update({k: u for k, u in _ELSEWHERE.items() if os.path.exists(_source(u))})
        _entry_points = found
    return _entry_points


def with_needs(wanted: Iterable[str]) -> List[str]:
    """The units and everything they need, what is needed first."""
    order: List[str] = []

    def add(unit):
        if unit in order:
            return
        for n in ((BASE_UNIT,) if unit != BASE_UNIT else ()) + tuple(NEEDS.get(unit, ())):
            add(n)
        if unit not in order:
            order.append(unit)
    for u in wanted:
        add(u)
    return order


def _writable(folder: str) -> bool:
    try:
        os.makedirs(folder, exist_ok=True)
        probe = os.path.join(folder, f".probe{os.getpid()}")
        with open(probe, "w"):
            pass
        os.remove(probe)
        return True
    except OSError:
        return False


def _build_dirs():
    in_tree = os.path.join(CSRC, "_build")
    tag = hashlib.sha1(CSRC.encode()).hexdigest()[:12]
    fallback = os.path.join(tempfile.gettempdir(), f"deliverance_amd_build_{os.getuid()}_{tag}")
    return in_tree, fallback


def _find_hipcc():
    for cand in (os.environ.get("HIPCC"), shutil.which("hipcc"), "/opt/rocm/bin/hipcc"):
        if cand and os.path.exists(cand):
            return cand
    return None


def _newest_source(unit: str) -> float:
    files = [_source(unit)] + glob.glob(os.path.join(CSRC, "*.h"))
    if unit in INCLUDES:
        files.append(_source(INCLUDES[unit]))
    return max(os.path.getmtime(f) for f in files)


def unit_path(unit: str) -> Optional[str]:
    """The unit's usable library, or None when it has to be compiled."""
    for d in _build_dirs():
        p = os.path.join(d, f"libda_{unit}.so")
        if os.path.exists(p) and os.path.getmtime(p) >= _newest_source(unit):
            return p
    return None


def missing(wanted: Optional[Iterable[str]] = None) -> List[str]:
    """Which of the units (all of them by default) are not built, with what they need."""
    return [u for u in with_needs(units() if wanted is None else wanted) if unit_path(u) is None]


def is_built() -> bool:
    return not missing()


def build(force: bool = False, verbose: bool = True, only: Optional[Sequence[str]] = None) -> str:
    """Compile every unit (or ``only`` those and what they need): the missing ones, or all of them with ``force``.
    Returns the folder of the libraries."""
    names = with_needs(units() if only is None else only)
    if not names or any(not os.path.exists(_source(u)) for u in names):
        raise KernelLibraryError(f"no HIP sources for {', '.join(names) or 'anything'} under {CSRC}")
    in_tree, fallback = _build_dirs()
    todo = names if force else [u for u in names if unit_path(u) is None]
    if not todo:
        return in_tree if os.path.isdir(in_tree) else fallback
    hipcc = _find_hipcc()
    if hipcc is None:
        raise KernelLibraryError(
            "the HIP kernels are not built and hipcc was not found (looked at $HIPCC, PATH and "
            "/opt/rocm/bin/hipcc); this engine has no other compute path")
    out_dir = in_tree if _writable(in_tree) else fallback
    if not _writable(out_dir):
        raise KernelLibraryError(f"cannot write the kernel libraries to {in_tree} or {fallback}")
    # one build at a time per folder: processes that start together in a fresh checkout would
    # otherwise write the same object files; whoever waited finds the libraries built
    with open(os.path.join(out_dir, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not force:
            todo = [u for u in names if unit_path(u) is None]
        if todo:
            _build_locked(hipcc, out_dir, todo, verbose)
    return out_dir


def _build_locked(hipcc: str, out_dir: str, todo: Sequence[str], verbose: bool) -> None:
    env = dict(os.environ)
    env.setdefault("HOME", out_dir)       # hipcc wants somewhere to keep its temporary files
    env.setdefault("TMPDIR", tempfile.gettempdir())
    t0 = time.time()

    def say(msg):
        if verbose:
            print(f"[deliverance_amd build] {msg}", file=sys.stderr, flush=True)

    def run(cmd, what):
        r = subprocess.run(cmd, capture_output=True, text=True, env=env)
        if r.returncode != 0:
            raise KernelLibraryError(f"{what} failed:\n{r.stdout}\n{r.stderr}")

    say(f"compiling {len(todo)} HIP sources for {ARCH} into {out_dir}")

    def compile_one(unit):
        obj = os.path.join(out_dir, unit + ".o")
        run([hipcc, *HIPCC_FLAGS, *EXTRA_FLAGS.get(unit, []), "-I", CSRC, "-c", _source(unit), "-o", obj], f"hipcc on {unit}.hip")
        tmp = os.path.join(out_dir, f".libda_{unit}.so.{os.getpid()}")
        run([hipcc, "-shared", "-fPIC", f"--offload-arch={ARCH}", obj, "-o", tmp], f"linking {unit}")
        os.replace(tmp, os.path.join(out_dir, f"libda_{unit}.so"))
        say(f"  {unit} done ({time.time() - t0:.0f}s)")

    # the long ones first
    order = sorted(todo, key=lambda u: -os.path.getsize(_source(u)))
    workers = max(1, min(len(order), int(os.environ.get("MAX_JOBS", "8")), 16))
    with ThreadPoolExecutor(max_workers=workers) as pool:
        list(pool.map(compile_one, order))
    say(f"built {len(todo)} in {time.time() - t0:.0f}s")


def ensure(wanted: Iterable[str], verbose: bool = True) -> None:
    """Compile what is missing of these units, side by side."""
    if _lib is None or isinstance(_lib, Library):
        build(force=False, verbose=verbose, only=list(wanted))


class Library:
    """The entry points of all units; a unit is loaded (and compiled, when it is missing) with its first entry point."""

    def __init__(self):
        self._handles: Dict[str, ctypes.CDLL] = {}

    def _open(self, unit: str) -> ctypes.CDLL:
        if unit not in self._handles:
            import torch  # noqa: F401  (loads libamdhip64 first: the units bind to the HIP runtime torch has loaded)
            chain = with_needs([unit])
            if any(unit_path(u) is None for u in chain):
                build(force=False, only=[unit])
            shared = {BASE_UNIT, *(n for ns in NEEDS.values() for n in ns)}
            for u in chain:
                if u in self._handles:
                    continue
                path = unit_path(u)
                try:
                    self._handles[u] = ctypes.CDLL(path, mode=ctypes.RTLD_GLOBAL if u in shared else ctypes.DEFAULT_MODE)
                except OSError as e:
                    raise KernelLibraryError(f"cannot load {path}: {e}") from None
        return self._handles[unit]

    def __getattr__(self, name: str):
        unit = entry_points().get(name) if name.startswith("da_") else None
        if unit is None:
            raise AttributeError(name)
        fn = getattr(self._open(unit), name)
        if name == "da_last_error":
            fn.restype = ctypes.c_char_p
        setattr(self, name, fn)             # found without this detour from now on
        return fn


def load() -> Library:
    global _lib
    if _lib is None:
        _lib = Library()
    return _lib
