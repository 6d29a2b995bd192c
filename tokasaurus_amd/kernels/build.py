"""Builds the gfx950 kernel libraries from ``tokasaurus_amd/csrc`` with hipcc.

There are three shared objects, loaded through ctypes (no Python headers, no torch
headers): ``core`` holds the kernels every model needs in either storage type,
``mfma`` the bfloat16 matrix-core kernels and ``library`` the calls of the matrix
product library (hipBLASLt) for many rows of bfloat16, both of which a 32-bit run
never loads and so never compiles.  A fresh checkout builds what it needs at its first call in
well under a minute.  ``ensure_built`` is what the loader calls: it compiles only
when no library matching the current sources exists, and prints a line per file
meanwhile.  The libraries live in ``tokasaurus_amd/kernels/_build``; when that
folder cannot be written (a checkout owned by someone else) they are built in a
folder of the user's own under the system's temporary folder.
"""

from __future__ import annotations

import hashlib
import os
import shutil
import subprocess
import sys
import tempfile
import time
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

CSRC = Path(__file__).resolve().parent.parent / "csrc"
IN_TREE_DIR = Path(__file__).resolve().parent / "_build"
GROUPS = {
    "core": ["errors.hip", "elementwise.hip", "attention_generic.hip", "gemm_generic.hip", "sample.hip", "step_io.hip",
             "stream_f32.hip", "attention_prepare.hip", "attention_tile_f32.hip", "delta_rule.hip", "routed_experts.hip", "gated_recurrence.hip", "linear_attention.hip", "linear_attention_chunks.hip", "state_space.hip"],
    "mfma": ["errors.hip", "attention_mfma.hip", "gemm_mfma.hip", "grouped_gemm.hip"],
    "library": ["errors.hip", "gemm_library.hip"],
}
# what a group's library is linked with beside the HIP runtime
LINK_FLAGS = {"library": ["-lhipblaslt"]}

ARCH = "gfx950"
# packed 32-bit float instructions are kept off for every kernel of this library
HIPCC_FLAGS = [
    f"--offload-arch={ARCH}",
    "-fvisibility=hidden",
    "-O3",
    "-fPIC",
    "-std=c++17",
    "-Wno-unused-result",
    "-Xclang",
    "-target-feature",
    "-Xclang",
    "-packed-fp32-ops",
]


# The attention kernel rescales its accumulators between matrix products: they stay in
# ordinary vector registers instead of moving to and from the accumulation registers.
# No NaN reaches its arithmetic (the scores of keys out of range, whatever their pages hold, are
# replaced by minus infinity and their values by zero bits before anything is computed from
# them, and every difference of two infinities is guarded), so a maximum need not first make
# its operands quiet numbers: an instruction less for every score, in a loop whose time goes
# to such instructions.
SOURCE_FLAGS = {"attention_mfma.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1", "-fno-honor-nans"]}


# A developer's knob: extra flags for every hipcc call.  Part of the digest,
# so a library built with it is not taken for one built without.
EXTRA_FLAGS = os.environ.get("TOKASAURUS_HIPCC_EXTRA", "").split()


class BuildError(RuntimeError):
    pass


def sources(group: str) -> list[Path]:
    return [CSRC / name for name in GROUPS[group]]


def _hipcc() -> str:
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not Path(exe).exists():
        raise BuildError("hipcc not found: the kernel library cannot be built on this machine")
    return exe


def _digest(group: str) -> str:
    h = hashlib.sha256()
    h.update(" ".join(HIPCC_FLAGS + EXTRA_FLAGS).encode())
    h.update(repr(sorted(SOURCE_FLAGS.items())).encode())
    h.update(" ".join(LINK_FLAGS.get(group, [])).encode())
    for p in sorted(CSRC.glob("*.h")) + sources(group):
        h.update(p.name.encode())
        h.update(p.read_bytes())
    return h.hexdigest()


def _writable(folder: Path) -> bool:
    try:
        folder.mkdir(parents=True, exist_ok=True)
        probe = folder / f".probe{os.getpid()}"
        probe.write_text("")
        probe.unlink()
        return True
    except OSError:
        return False


def build_dir() -> Path:
    """The in-tree folder, or a folder of the user's own when that one cannot be written."""
    if _writable(IN_TREE_DIR):
        return IN_TREE_DIR
    own = Path(tempfile.gettempdir()) / f"tokasaurus_amd_build_{os.getuid()}"
    if not _writable(own):
        raise BuildError(f"neither {IN_TREE_DIR} nor {own} can be written: nowhere to build the kernel library")
    return own


def library_name(group: str) -> str:
    return f"libtokasaurus_{group}.so"


def find_current(group: str) -> Path | None:
    """A library of this group built from the current sources, wherever it was built."""
    digest = _digest(group)
    for folder in (IN_TREE_DIR, Path(tempfile.gettempdir()) / f"tokasaurus_amd_build_{os.getuid()}"):
        lib, stamp = folder / library_name(group), folder / f"stamp_{group}"
        try:
            if lib.is_file() and stamp.is_file() and stamp.read_text().strip() == digest:
                return lib
        except OSError:
            continue
    return None


def _say(msg: str) -> None:
    print(f"[tokasaurus_amd build] {msg}", file=sys.stderr, flush=True)


def _compile_one(hipcc: str, src: Path, obj: Path) -> tuple[Path, float]:
    t0 = time.time()
    cmd = [hipcc, *HIPCC_FLAGS, *EXTRA_FLAGS, *SOURCE_FLAGS.get(src.name, []), "-I", str(CSRC), "-c", str(src), "-o", str(obj)]
    proc = subprocess.run(cmd, capture_output=True, text=True)
    if proc.returncode != 0:
        raise BuildError(f"hipcc failed on {src.name}:\n{proc.stderr[-4000:]}")
    return src, time.time() - t0


def build_group(group: str, jobs: int | None = None) -> Path:
    """Compile the sources of one group and link its library."""
    hipcc = _hipcc()
    folder = build_dir()
    srcs = sources(group)
    missing = [s.name for s in srcs if not s.is_file()]
    if missing:
        raise BuildError(f"kernel sources missing under {CSRC}: {missing}")
    jobs = jobs or min(len(srcs), int(os.environ.get("MAX_JOBS", "8")), 16)
    _say(f"compiling the {group} kernels ({len(srcs)} HIP sources) for {ARCH} with {jobs} jobs into {folder}")
    objs = [folder / (f"{group}_{s.stem}.{os.getpid()}.o") for s in srcs]
    t0 = time.time()
    try:
        with ThreadPoolExecutor(max_workers=jobs) as pool:
            futures = [pool.submit(_compile_one, hipcc, s, o) for s, o in zip(srcs, objs)]
            for fut in futures:
                src, dt = fut.result()
                _say(f"  {src.name} done in {dt:.1f}s")
        tmp = folder / (library_name(group) + f".tmp{os.getpid()}")
        link = [hipcc, f"--offload-arch={ARCH}", "-shared", "-fPIC", "-o", str(tmp), *map(str, objs), *LINK_FLAGS.get(group, [])]
        proc = subprocess.run(link, capture_output=True, text=True)
        if proc.returncode != 0:
            raise BuildError(f"link failed:\n{proc.stderr[-4000:]}")
        os.replace(tmp, folder / library_name(group))
        (folder / f"stamp_{group}").write_text(_digest(group) + "\n")
    finally:
        for o in objs:
            try:
                o.unlink()
            except OSError:
                pass
    _say(f"built {folder / library_name(group)} in {time.time() - t0:.1f}s")
    return folder / library_name(group)


def build(force: bool = True) -> list[Path]:
    """Every group.  ``force=False`` skips a group whose library matches the current sources."""
    out = []
    for group in GROUPS:
        current = None if force else find_current(group)
        out.append(current or build_group(group))
    return out


def ensure_built(group: str) -> Path:
    """The library of a group for the current sources, compiling it if it is not there."""
    current = find_current(group)
    if current is not None:
        return current
    if (IN_TREE_DIR / library_name(group)).is_file():
        _say(f"the built {group} library does not match the sources; building again")
    return build_group(group)


if __name__ == "__main__":
    build(force=True)
