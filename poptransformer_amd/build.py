"""Build of the HIP libraries with hipcc for gfx950: libpoptransformer_hip.so from ``csrc/*.hip``, and
libpoptransformer_hybrid.so (decoders with recurrent layers and a 32-bit residual) from ``csrc/hybrid/*.hip``.

The reference builds its ``custom_ops.so`` with ``popc`` (codelets) and ``g++ -shared -lpopart
-lpoplar`` (/root/reference Makefile:1-37); this is the counterpart for MI355X.  A library is
written next to this package so that it is found in-tree and travels with the source tree.  A caller that needs
one of them only (``build(libraries=("hybrid",))``) compiles no more than that one.
"""
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
OBJ_DIR = os.path.join(HERE, "build")
LIB_PATH = os.path.join(HERE, "libpoptransformer_hip.so")

HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-fno-fast-math", "-ffp-contract=off",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-Wno-unused-command-line-argument",
]


def _hipcc():
    for cand in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if cand and (os.path.isabs(cand) and os.path.exists(cand) or not os.path.isabs(cand)):
            return cand
    raise RuntimeError("hipcc not found")


INCLUDE = os.path.join(HERE, "..", "include")
# name -> (directory of the sources, library)
LIBRARIES = {"hip": (CSRC, LIB_PATH),
             "hybrid": (os.path.join(CSRC, "hybrid"), os.path.join(HERE, "libpoptransformer_hybrid.so"))}


def sources(directory=CSRC):
    return sorted(os.path.join(directory, f) for f in os.listdir(directory) if f.endswith(".hip"))


def _headers():
    return [os.path.join(d, f) for d in (CSRC, os.path.join(CSRC, "hybrid"), INCLUDE) for f in os.listdir(d) if f.endswith(".h")]


def _compile(src, force):
    obj = os.path.join(OBJ_DIR, os.path.relpath(src, CSRC)[:-4].replace(os.sep, "_") + ".o")
    if not force and os.path.exists(obj) and all(os.path.getmtime(obj) > os.path.getmtime(d) for d in _headers() + [src]):
        return obj
    cmd = [_hipcc(), *HIPCC_FLAGS, "-c", src, "-o", obj]
    proc = subprocess.run(cmd, capture_output=True, text=True)
    if proc.returncode != 0:
        raise RuntimeError(f"hipcc failed for {src}:\n{proc.stdout}\n{proc.stderr}")
    return obj


def build(force=True, jobs=None, verbose=False, libraries=tuple(LIBRARIES)):
    """Compile the kernels of `libraries` and link them. Returns the path of the last one."""
    os.makedirs(OBJ_DIR, exist_ok=True)
    jobs = jobs or min(8, os.cpu_count() or 1)
    work = [(name, src) for name in libraries for src in sources(LIBRARIES[name][0])]
    with ThreadPoolExecutor(max_workers=jobs) as ex:
        objs = list(ex.map(lambda w: _compile(w[1], force), work))
    path = None
    for name in libraries:
        path = LIBRARIES[name][1]
        mine = [o for o, w in zip(objs, work) if w[0] == name]
        part = f"{path}.{os.getpid()}"            # linked aside and moved: a reader never sees half a library
        cmd = [_hipcc(), "--offload-arch=gfx950", "-shared", "-fPIC", "-Wl,-Bsymbolic", "-o", part, *mine]
        proc = subprocess.run(cmd, capture_output=True, text=True)
        if proc.returncode != 0:
            raise RuntimeError(f"link failed:\n{proc.stdout}\n{proc.stderr}")
        os.replace(part, path)
        if verbose:
            print(f"built {path}", file=sys.stderr)
    return path


if __name__ == "__main__":
    build(force="--force" in sys.argv, verbose=True)
