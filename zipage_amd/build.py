"""Build the HIP libraries (gfx950) in-tree with hipcc.

Run as ``python -m zipage_amd.build``.  Shared objects with a plain C ABI, none linked against
torch: ``libzipage_hip.so`` (``include/zipage_hip.h``: the compression path and the kernels of the
models that use it) and, for the other models, ``libzipage_models.so``, ``libzipage_latent.so``,
``libzipage_grouped.so``, ``libzipage_recurrent.so``, ``libzipage_linear.so`` and ``libzipage_moe.so``
(``include/zipage_models.h``), so that a model compiles only what it runs.
"""
from __future__ import annotations

import os
import shutil
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB = os.path.join(HERE, "libzipage_hip.so")
MODELS_LIB = os.path.join(HERE, "libzipage_models.so")
LATENT_LIB = os.path.join(HERE, "libzipage_latent.so")
GROUPED_LIB = os.path.join(HERE, "libzipage_grouped.so")
RECURRENT_LIB = os.path.join(HERE, "libzipage_recurrent.so")
LINEAR_LIB = os.path.join(HERE, "libzipage_linear.so")
MOE_LIB = os.path.join(HERE, "libzipage_moe.so")

# packed fp32 VALU ops are disabled on purpose (some forms misbehave on this fleet)
BASE_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-Wno-unused-command-line-argument",
]
# keep a*b+c as two roundings: the compression stages restate torch ops that round after each op
FLAGS = BASE_FLAGS + ["-ffp-contract=off"]

# sources of the model-side libraries, beside the error reporting; the rest is the compression library
MODEL_SOURCES = {
    MODELS_LIB: ("residual.hip", "runs.hip"),
    LATENT_LIB: ("latent.hip",),
    GROUPED_LIB: ("grouped.hip",),
    RECURRENT_LIB: ("mlstm.hip", "mlstm_runs.hip", "delta.hip", "delta_runs.hip"),
    LINEAR_LIB: ("linear.hip", "linear_runs.hip"),
    MOE_LIB: ("moe.hip",),
}
COMMON_SOURCES = ("runtime.hip",)
LIBS = (LIB, *MODEL_SOURCES)


def sources(lib: str = LIB) -> list[str]:
    if lib in MODEL_SOURCES:
        names = [*MODEL_SOURCES[lib], *COMMON_SOURCES]
    else:
        others = {f for fs in MODEL_SOURCES.values() for f in fs}
        names = [f for f in os.listdir(CSRC) if f.endswith(".hip") and f not in others]
    return sorted(os.path.join(CSRC, f) for f in names)


def _run(cmd, verbose):
    if verbose:
        print(" ".join(cmd), flush=True)
    proc = subprocess.run(cmd, capture_output=True, text=True)
    err = "\n".join(l for l in proc.stderr.splitlines()
                    if "is not a recognized feature for this target" not in l)
    if proc.returncode != 0:
        raise RuntimeError(f"hipcc failed ({proc.returncode}):\n{proc.stdout}\n{err}")
    if verbose and err.strip():
        print(err, file=sys.stderr)


def build(verbose: bool = True, jobs: int | None = None, libs: tuple[str, ...] = LIBS) -> str:
    """Compile the sources of ``libs`` to object files (in parallel) and link the shared objects."""
    from concurrent.futures import ThreadPoolExecutor
    hipcc = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    extra = os.environ.get("ZP_EXTRA_HIPCC_FLAGS", "").split()
    work, links = [], []
    for lib in libs:
        models = lib in MODEL_SOURCES
        objdir = os.path.join(HERE, "build", os.path.basename(lib)[len("libzipage_"):-3] if models else "")
        os.makedirs(objdir, exist_ok=True)
        objs = []
        for src in sources(lib):
            obj = os.path.join(objdir, os.path.basename(src)[:-4] + ".o")
            work.append([hipcc, *(BASE_FLAGS if models else FLAGS), *extra, "-c", src, "-o", obj])
            objs.append(obj)
        links.append((lib, objs))
    jobs = jobs or min(len(work), os.cpu_count() or 1, 16)
    with ThreadPoolExecutor(max_workers=jobs) as pool:
        list(pool.map(lambda cmd: _run(cmd, verbose), work))
    for lib, objs in links:
        _run([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC", *objs, "-o", lib + ".tmp"], verbose)
        os.replace(lib + ".tmp", lib)
    return libs[0]


def ensure(*libs: str) -> None:
    """Build those of ``libs`` that are not there yet (one process at a time)."""
    if not all(os.path.exists(lib) for lib in libs):
        import fcntl
        os.makedirs(os.path.join(HERE, "build"), exist_ok=True)
        with open(os.path.join(HERE, "build", ".lock"), "w") as lock:
            fcntl.flock(lock, fcntl.LOCK_EX)
            missing = tuple(lib for lib in libs if not os.path.exists(lib))
            if missing:
                build(verbose=False, libs=missing)


if __name__ == "__main__":
    print(build())
