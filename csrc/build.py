"""Build the CDNA4 kernel libraries in-tree.

hipcc cross-compiles gfx950 without a GPU, so this runs in CPU-only CI.
The resulting shared libraries live inside the package (they travel with
the repo snapshot to GPU boxes; they are git-ignored so history stays
source-only).  One library per mechanism, so a model compiles only what it
launches:

    llmops   dense/MoE transformer kernels, sampler, xGMI collectives

and the paged mixed-batch kernels of the layer-list designs:

    linear     embedding, norms and linears around an fp32 residual
    latent     attention over a cache of latents
    gqa        grouped-query attention
    mlstm      matrix-memory LSTM
    mingru     gated recurrence of single tokens' gates
    ssd        state-space recurrence behind a short convolution
    rglru      gated linear recurrence behind a short convolution
    lightning  linear attention with a decay per head
    moe        routed experts
"""

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CSRC = os.path.join(ROOT, "csrc")
PKG = os.path.join(ROOT, "llm_np_cp_amd")
LIBS = {
    "llmops": ["llm_ops.hip", "xgmi_comm.hip"],
    "linear": ["linear.hip"],
    "latent": ["latent_attn.hip"],
    "gqa": ["gqa_attn.hip"],
    "mlstm": ["mlstm.hip"],
    "mingru": ["mingru.hip"],
    "ssd": ["ssd.hip"],
    "rglru": ["rglru.hip"],
    "lightning": ["lightning.hip"],
    "moe": ["moe.hip"],
}
HEADERS = ["attn_split.h", "common.h", "gemm_tile.h", "hybrid.h", "mingru.h",
           "moe.h"]
# Packed fp32 VALU forms are kept out of all device code: some of them
# have returned wrong results on this hardware.  (The host pass warns that
# it does not know the feature.)
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC",
         "-Wno-unused-value", "-Wno-unused-result",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def lib_path(name: str) -> str:
    return os.path.join(PKG, f"_lib{name}.so")


def _run(cmd, verbose: bool):
    if verbose:
        print("+", " ".join(cmd), flush=True)
    p = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT,
                       text=True)
    if p.returncode != 0:
        sys.stderr.write(p.stdout)
        raise RuntimeError(f"hipcc failed ({p.returncode}): {' '.join(cmd)}")


def _replace_from(tmp: str, cmd, out: str, verbose: bool):
    """Run cmd writing tmp, then move it to out (concurrent builders and
    readers never see half a file)."""
    try:
        _run(cmd, verbose)
        os.replace(tmp, out)
    finally:
        if os.path.exists(tmp):
            os.unlink(tmp)


def _stale(out: str, deps) -> bool:
    return not os.path.exists(out) or any(
        os.path.getmtime(d) > os.path.getmtime(out) for d in deps)


def _deps(name: str):
    return [os.path.join(CSRC, f) for f in LIBS[name] + HEADERS]


def needs_rebuild(name: str = "llmops") -> bool:
    return _stale(lib_path(name), _deps(name))


def build(verbose: bool = True, names=None, force: bool = True):
    """Compile the named libraries (default: all) and return their paths.
    Objects land in build/ and are compiled in parallel."""
    names = list(names or LIBS)
    objdir = os.path.join(ROOT, "build", "obj")
    os.makedirs(objdir, exist_ok=True)
    hdrs = [os.path.join(CSRC, h) for h in HEADERS]
    jobs, objs = [], {n: [] for n in names}
    for n in names:
        for src in LIBS[n]:
            path = os.path.join(CSRC, src)
            obj = os.path.join(objdir, src + ".o")
            objs[n].append(obj)
            if force or _stale(obj, [path] + hdrs):
                jobs.append((path, obj))

    def compile_one(job):
        path, obj = job
        tmp = f"{obj}.{os.getpid()}.o"
        _replace_from(tmp, ["hipcc", *FLAGS, "-c", path, "-o", tmp], obj,
                      verbose)

    workers = min(8, max(1, len(jobs)))
    with ThreadPoolExecutor(workers) as ex:
        list(ex.map(compile_one, jobs))
    outs = []
    for n in names:
        out = lib_path(n)
        tmp = f"{out}.{os.getpid()}.tmp"
        _replace_from(tmp, ["hipcc", "--offload-arch=gfx950", "-shared",
                            *objs[n], "-o", tmp], out, verbose)
        outs.append(out)
    return outs


def ensure_built(verbose: bool = False, names=None):
    """Build what is missing or older than its sources."""
    names = list(names or LIBS)
    stale = [n for n in names if needs_rebuild(n)]
    if stale:
        build(verbose=verbose, names=stale, force=False)
    return [lib_path(n) for n in names]


if __name__ == "__main__":
    for _p in build():
        print("built", _p)
