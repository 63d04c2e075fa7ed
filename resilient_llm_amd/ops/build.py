"""In-tree build of the gfx950 HIP extension.

Direct ``hipcc`` invocation (no ninja, no JIT cache): the resulting
``_rlli_hip.so`` sits next to this file, ships to the GPU box with the
repo snapshot, and loads via ``torch.ops.load_library`` — so a fresh box
never recompiles.  Incremental: each translation unit recompiles only
when its mtime (or a header's) is newer than its object file.

Usage: python -m resilient_llm_amd.ops.build [--force]
"""

from __future__ import annotations

import concurrent.futures as cf
import os
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950")
# Host-side sanitizers for the extension: RLLI_ASAN=1 /
# RLLI_TSAN=1 add -fsanitize to host code (device code unaffected).
# Sanitized builds go to their OWN objects + .so so they never clobber
# the production artifact that ships to GPU boxes.
_SAN = ("asan" if os.environ.get("RLLI_ASAN") == "1" else
        "tsan" if os.environ.get("RLLI_TSAN") == "1" else "")
SAN_FLAGS = {"asan": ["-Xarch_host", "-fsanitize=address"],
             "tsan": ["-Xarch_host", "-fsanitize=thread"], "": []}[_SAN]
BUILD = os.path.join(HERE, "build" + (f"-{_SAN}" if _SAN else ""))

# Libraries, so that a process compiles and loads what its model needs:
# rlli_hip has the Llama-family kernels and the sampler, rlli_attn paged
# softmax attention in its variants, rlli_mix residual streams, windowed
# prompt attention and mixture of experts, rlli_blk residual blocks and short
# convolutions, rlli_rec linear recurrences, rlli_lat latent attention.
LIBRARIES = {
    "rlli_hip": [
        "ext.cpp",
        "lt_gemm.cpp",
        "rmsnorm.hip",
        "silu_mul.hip",
        "rope_kv.hip",
        "decode_attn.hip",
        "prefill_attn.hip",
        "prefill_mfma.hip",
        "prefill_paged.hip",
        "sampling.hip",
        "skinny_gemm.hip",
        "skinny2.hip",
        "streamprobe.hip",
    ],
    "rlli_attn": [
        "ext_attn.cpp",
        "window_attn.hip",
        "diff_attn.hip",
        "expanded_attn.hip",
    ],
    "rlli_mix": [
        "ext_mix.cpp",
        "hyper.hip",
        "window_prefill.hip",
        "moe.hip",
    ],
    "rlli_blk": [
        "ext_blk.cpp",
        "block.hip",
    ],
    "rlli_rec": [
        "ext_rec.cpp",
        "gla.hip",
        "delta.hip",
        "mlstm.hip",
        "rec_scan.hip",
    ],
    "rlli_lat": [
        "ext_lat.cpp",
        "latent.hip",
    ],
}
_ACT = ["common.h", "act.h", "ext_common.h"]
_ATTN = _ACT + ["attn.h", "attn_rows.h", "ext_window.h"]
HEADERS = {"rlli_hip": ["common.h", "kernels.h"],
           "rlli_attn": _ATTN,
           "rlli_mix": _ATTN + ["mix.h"],
           "rlli_blk": _ACT + ["blk.h"],
           "rlli_rec": _ACT + ["rec.h", "rec_math.h"],
           "rlli_lat": _ATTN + ["lat.h"]}
# some packed f32 instruction forms have returned wrong results on this
# hardware; keep the compiler from forming them
CODEGEN = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def so_path(lib: str) -> str:
    return os.path.join(HERE, f"_{lib}{'_' + _SAN if _SAN else ''}.so")


OUT_SO = so_path("rlli_hip")


def _torch_flags() -> tuple[list[str], list[str]]:
    import torch
    import torch.utils.cpp_extension as ce
    includes = [f"-I{p}" for p in ce.include_paths()]
    libs = [f"-L{p}" for p in ce.library_paths()]
    libs += ["-ltorch", "-ltorch_cpu", "-lc10", "-ltorch_hip", "-lc10_hip",
             "-lamdhip64", "-lhipblaslt"]
    abi = int(torch._C._GLIBCXX_USE_CXX11_ABI)
    includes.append(f"-D_GLIBCXX_USE_CXX11_ABI={abi}")
    return includes, libs


def _deps(lib: str, src: str) -> list[str]:
    return [os.path.join(CSRC, f) for f in [src] + HEADERS[lib]] \
        + [os.path.abspath(__file__)]


def _compile_one(lib: str, src: str, includes: list[str],
                 force: bool) -> str:
    obj = os.path.join(BUILD, src.replace("/", "_") + ".o")
    if not force and os.path.exists(obj) and all(
            os.path.getmtime(d) <= os.path.getmtime(obj)
            for d in _deps(lib, src)):
        return obj
    cmd = (["hipcc", f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC",
            "-DNDEBUG"] + CODEGEN
           + ["-c", os.path.join(CSRC, src), "-o", obj, f"-I{CSRC}"]
           + SAN_FLAGS + includes)
    print("  hipcc -c", src, flush=True)
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"hipcc failed on {src}:\n{r.stderr[-8000:]}")
    return obj


def _link(lib: str, objs: list[str], libs: list[str], force: bool,
          verbose: bool) -> str:
    out = so_path(lib)
    if not force and os.path.exists(out) and all(
            os.path.getmtime(o) <= os.path.getmtime(out) for o in objs):
        return out
    # link aside and rename: a process that loads meanwhile never sees
    # half a library
    tmp = f"{out}.tmp{os.getpid()}"
    cmd = (["hipcc", f"--offload-arch={ARCH}", "-shared", "-fPIC",
            "-o", tmp] + SAN_FLAGS + objs + libs)
    if verbose:
        print("  hipcc -shared ->", os.path.basename(out), flush=True)
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"link failed:\n{r.stderr[-8000:]}")
    os.replace(tmp, out)
    return out


def build(force: bool = False, verbose: bool = True,
          libs: tuple = tuple(LIBRARIES)) -> str:
    """Compile ``libs`` (incrementally unless ``force``); returns the path
    of the first one."""
    os.makedirs(BUILD, exist_ok=True)
    includes, link = _torch_flags()
    work = [(lib, src) for lib in libs for src in LIBRARIES[lib]]
    jobs = min(int(os.environ.get("MAX_JOBS", "8")), 16, len(work))
    with cf.ThreadPoolExecutor(max_workers=max(1, jobs)) as ex:
        objs = list(ex.map(lambda w: _compile_one(*w, includes, force), work))
    for lib in libs:
        _link(lib, [o for (n, _), o in zip(work, objs) if n == lib], link,
              force, verbose)
    return so_path(libs[0])


def ensure(libs: tuple) -> None:
    """Build those of ``libs`` that are missing or older than a source."""
    def stale(lib):
        out = so_path(lib)
        return not os.path.exists(out) or any(
            os.path.getmtime(d) > os.path.getmtime(out)
            for src in LIBRARIES[lib] for d in _deps(lib, src))
    todo = tuple(lib for lib in libs if stale(lib))
    if todo:
        build(libs=todo)


if __name__ == "__main__":
    build(force="--force" in sys.argv)
    print("built", ", ".join(map(so_path, LIBRARIES)))
