"""In-tree build of the CDNA4 kernel libraries.

Hand-driven hipcc (no hipify, no CUDA shims): ``csrc/*.hip`` is gfx950
device code compiled with ``--offload-arch=gfx950`` and linked into shared
libraries loaded via ctypes.  Built IN-TREE so the .so files travel with
the source tree.

Two libraries, so that a serving process compiles only what it runs:

* ``libnxd_ops.so``      every ``csrc/*.hip`` — training kernels and the
                         batch-synchronous inference kernels,
* ``libnxd_serving.so``  every ``csrc/serving/*.hip`` — the ragged-batch
                         kernels of the serving engine.
"""

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

_THIS = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(_THIS, "csrc")
LIB = os.path.join(_THIS, "libnxd_ops.so")
SERVING_LIB = os.path.join(_THIS, "libnxd_serving.so")

GROUPS = {
    "ops": (CSRC, LIB),
    "serving": (os.path.join(CSRC, "serving"), SERVING_LIB),
}

HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
ARCH = os.environ.get("NXDA_GPU_ARCH", "gfx950")

# packed-FP32 instruction forms are off for all device code (the host pass
# warns that it does not know the feature; the warning is silenced)
FLAGS = [f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC",
         "-ffp-contract=fast",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _listed(folder, ext):
    return sorted(os.path.join(folder, f) for f in os.listdir(folder)
                  if f.endswith(ext))


def _sources(group="ops"):
    return _listed(GROUPS[group][0], ".hip")


def _headers(group):
    folder = GROUPS[group][0]
    return _listed(CSRC, ".h") + (_listed(folder, ".h")
                                  if folder != CSRC else [])


def _needs_build(group="ops"):
    lib = GROUPS[group][1]
    if not os.path.exists(lib):
        return True
    lib_mtime = os.path.getmtime(lib)
    return any(os.path.getmtime(s) > lib_mtime
               for s in _sources(group) + _headers(group))


def _run(cmd, verbose):
    if verbose:
        print("[nxd_ops]", " ".join(cmd), file=sys.stderr, flush=True)
    r = subprocess.run(cmd, stdout=subprocess.PIPE,
                       stderr=subprocess.STDOUT, text=True)
    out = "\n".join(l for l in r.stdout.splitlines()
                    if "packed-fp32-ops" not in l)
    if out.strip() and (verbose or r.returncode):
        print(out, file=sys.stderr, flush=True)
    if r.returncode:
        raise RuntimeError(f"hipcc failed ({r.returncode}): {' '.join(cmd)}")


def build_group(group: str, force: bool = False, verbose: bool = True) -> str:
    """Compile one library; its sources compile in parallel.  The finished
    library is renamed into place, so a concurrent reader never sees half
    of one."""
    lib = GROUPS[group][1]
    if not force and not _needs_build(group):
        return lib
    jobs = int(os.environ.get("MAX_JOBS", "8"))
    tmp = f"{lib}.{os.getpid()}"
    objs, cmds = [], []
    for s in _sources(group):
        o = f"{s[:-len('.hip')]}.{os.getpid()}.o"
        objs.append(o)
        cmds.append([HIPCC, *FLAGS, "-I", CSRC, "-c", s, "-o", o])
    try:
        with ThreadPoolExecutor(max_workers=max(1, min(jobs, 16))) as ex:
            list(ex.map(lambda c: _run(c, verbose), cmds))
        _run([HIPCC, f"--offload-arch={ARCH}", "-shared", "-fPIC", "-o", tmp,
              *objs], verbose)
        os.replace(tmp, lib)
    finally:
        for f in objs + [tmp]:
            if os.path.exists(f):
                os.unlink(f)
    return lib


def build(force: bool = False, verbose: bool = True) -> str:
    for group in GROUPS:
        build_group(group, force, verbose)
    return LIB


if __name__ == "__main__":
    build(force="--force" in sys.argv)
