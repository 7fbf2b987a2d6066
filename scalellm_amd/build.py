"""Build the C-ABI HIP kernel libraries in-tree with hipcc for gfx950.

    python -m scalellm_amd.build                      # incremental, every library
    python -m scalellm_amd.build --force
    python -m scalellm_amd.build --library latent     # one library only

  hip     csrc/*.hip         -> csrc/libslm_hip.so      int4 / 8-bit linears, paged MHA, all-reduce
  latent  csrc/latent/*.hip  -> csrc/libslm_latent.so   dense 16- / 32-bit path, latent attention
  mixers  csrc/mixers/*.hip  -> csrc/libslm_mixers.so   windowed attention with a sink, recurrent layers

The .so files are git-ignored.
"""
from __future__ import annotations

import contextlib
import fcntl
import glob
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
ROOT = os.path.dirname(HERE)
INCLUDE = os.path.join(ROOT, "include")
OBJ_DIR = os.path.join(CSRC, "build")
LIB = os.path.join(CSRC, "libslm_hip.so")
LATENT_LIB = os.path.join(CSRC, "libslm_latent.so")
MIXERS_LIB = os.path.join(CSRC, "libslm_mixers.so")
# library -> (source folder, result)
LIBRARIES = {"hip": (CSRC, LIB), "latent": (os.path.join(CSRC, "latent"), LATENT_LIB),
             "mixers": (os.path.join(CSRC, "mixers"), MIXERS_LIB)}
ARCH = "gfx950"

HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
CXXFLAGS = [
    f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC", "-fvisibility=hidden",
    "-fno-gpu-rdc", "-Wall", "-Wno-unused-function", f"-I{INCLUDE}", f"-I{CSRC}",
    # no packed fp32 arithmetic: some forms of it give wrong results now and then on this hardware
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
]
# (the host pass does not know the feature and says so, once per file)
_HARMLESS = ("'-packed-fp32-ops' is not a recognized feature",)


def _sources(folder: str):
    return sorted(glob.glob(os.path.join(folder, "*.hip")))


def _deps_mtime(folder: str):
    hdrs = [h for d in {folder, CSRC, INCLUDE, os.path.join(CSRC, "latent") if folder != CSRC else CSRC} for h in glob.glob(os.path.join(d, "*.h"))]
    return max(os.path.getmtime(h) for h in hdrs)


def _file_flags(src: str):
    """Extra hipcc flags a source file asks for on a `// hipcc-flags: ...` line in its header."""
    flags = []
    with open(src) as f:
        for i, line in enumerate(f):
            if i > 80:
                break
            if line.startswith("// hipcc-flags:"):
                flags += line.split(":", 1)[1].split()
    return flags


def _compile(src: str, force: bool) -> str:
    folder = os.path.dirname(src)
    prefix = "" if folder == CSRC else os.path.basename(folder) + "_"
    obj = os.path.join(OBJ_DIR, prefix + os.path.basename(src) + ".o")
    newest = max(os.path.getmtime(src), _deps_mtime(folder))
    if force or not os.path.exists(obj) or os.path.getmtime(obj) < newest:
        cmd = [HIPCC, *CXXFLAGS, *_file_flags(src), "-c", src, "-o", obj]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed for {src}:\n{r.stdout}\n{r.stderr}")
        noise = "\n".join(line for line in r.stderr.splitlines() if line and not any(h in line for h in _HARMLESS))
        if noise:
            sys.stderr.write(noise + "\n")
    return obj


@contextlib.contextmanager
def _locked():
    """One build at a time in a checkout (several processes may find the libraries missing at once)."""
    os.makedirs(OBJ_DIR, exist_ok=True)
    with open(os.path.join(OBJ_DIR, ".lock"), "w") as f:
        fcntl.flock(f, fcntl.LOCK_EX)
        yield


def build(force: bool = False, verbose: bool = True, library: str = "") -> str:
    """Compile what is out of date.  library: one of LIBRARIES, or "" for all; the path of the library (all:
    of libslm_hip.so) is returned."""
    names = [library] if library else list(LIBRARIES)
    with _locked():
        work = {n: _sources(LIBRARIES[n][0]) for n in names}
        if not all(work.values()):
            raise RuntimeError("no .hip sources found")
        srcs = [s for n in names for s in work[n]]
        with ThreadPoolExecutor(max_workers=min(8, len(srcs))) as ex:
            objs = dict(zip(srcs, ex.map(lambda s: _compile(s, force), srcs)))
        for n in names:
            lib = LIBRARIES[n][1]
            mine = [objs[s] for s in work[n]]
            if force or not os.path.exists(lib) or any(os.path.getmtime(o) > os.path.getmtime(lib) for o in mine):
                tmp = lib + ".tmp"
                subprocess.check_call([HIPCC, f"--offload-arch={ARCH}", "-shared", "-fPIC", "-o", tmp, *mine])
                os.replace(tmp, lib)
                if verbose:
                    print(f"[scalellm_amd.build] linked {lib}")
    return LIBRARIES[library or "hip"][1]


def ensure(library: str) -> str:
    """The built library, compiled now if nothing is there yet."""
    lib = LIBRARIES[library][1]
    return lib if os.path.exists(lib) else build(verbose=False, library=library)


if __name__ == "__main__":
    _only = sys.argv[sys.argv.index("--library") + 1] if "--library" in sys.argv else ""
    build(force="--force" in sys.argv, library=_only)
