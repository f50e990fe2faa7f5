"""Build recipe for the gfx950 shared objects (no cmake, no JIT cache).

    python mini-sglang_amd/build.py            # build what is stale
    python mini-sglang_amd/build.py --force

Outputs (git-ignored, shipped to the GPU box by gpurun because they are in-tree):
    mini-sglang_amd/lib/libmsgl_hip.so    every kernel + host helpers   (include/msgl_hip.h)
    mini-sglang_amd/lib/libmsgl_comm.so   RCCL communicator             (links librccl)
    mini-sglang_amd/lib/libmsgl_gemm.so   projection GEMMs + tuner      (links libhipblaslt)
    mini-sglang_amd/lib/libmsgl_mix.so    sequence-mixing kernels       (include/msgl_mix.h; no library dependency)

`build_all(only=("mix", "gemm"))` builds a subset: a model needs the libraries its layers call, not all of them.

hipcc cross-compiles for gfx950 without a GPU, so this also runs in the build container.
"""
from __future__ import annotations

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

ROOT = Path(__file__).resolve().parent
CSRC = ROOT / "csrc"
LIB = ROOT / "lib"
OBJ = ROOT / "build"
INCLUDE = ROOT.parent / "include"
ROCM = Path(os.environ.get("ROCM_PATH", "/opt/rocm"))
HIPCC = os.environ.get("HIPCC", str(ROCM / "bin" / "hipcc"))
ARCH = "gfx950"

HIP_SOURCES = [
    "host.cpp",
    "radix.cpp",
    "store_index.hip",
    "norm_rope_act.hip",
    "attn_decode.hip",
    "attn_prefill.hip",
    "sampling.hip",
    "gemm_skinny.hip",
    "gemm_rowstream.hip",
    "gemm_wstream.hip",
    "gemm_m256.hip",
    "gemm_g3.hip",
    "gemm_ro.hip",
    "comm_p2p.hip",
]
MIX_SOURCES = ["seqmix.hip", "mix_delta.hip", "mix_par.hip", "mix_scan.hip", "mix_streams.hip", "mix_sandwich.hip"]
COMM_SOURCES = ["comm.cpp"]
GEMM_SOURCES = ["gemm.cpp"]

COMMON_FLAGS = [
    "-O3",
    "-std=c++17",
    "-fPIC",
    f"--offload-arch={ARCH}",
    "-Wall",
    "-Wno-unused-function",
    "-Wno-inline-asm",
    "-I",
    str(INCLUDE),
]
if os.environ.get("MSGL_PREFILL_DIAG") == "1":  # timing-only ablation variants of the prefill kernels (tools/prefill_ablate.py)
    COMMON_FLAGS.append("-DMSGL_PREFILL_DIAG")


def _stale(out: Path, deps: list[Path]) -> bool:
    if not out.exists():
        return True
    t = out.stat().st_mtime
    return any(d.stat().st_mtime > t for d in deps if d.exists())


def _run(cmd: list[str]) -> None:
    proc = subprocess.run(cmd, capture_output=True, text=True)
    if proc.returncode != 0:
        sys.stderr.write(" ".join(cmd) + "\n" + proc.stdout + proc.stderr)
        raise RuntimeError(f"build step failed: {cmd[-1]}")
    if proc.stderr.strip():
        sys.stderr.write(proc.stderr)


# fp32 arithmetic stays scalar: no packed two-lane fp32 instructions in any kernel (a device-pass flag; the host pass says it does
# not know the feature, which is harmless)
KERNEL_FLAGS = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _compile(src: Path, force: bool) -> Path:
    obj = OBJ / (src.name + ".o")
    headers = list(CSRC.glob("*.h")) + list(INCLUDE.glob("*.h"))
    if force or _stale(obj, [src] + headers):
        extra = KERNEL_FLAGS if src.suffix == ".hip" else []
        _run([HIPCC, *COMMON_FLAGS, *extra, "-x", "hip", "-c", str(src), "-o", str(obj)])
    return obj


def build_all(force: bool = False, verbose: bool = True, only=None) -> dict[str, Path]:
    """Build the shared objects named in `only` (default: all of "hip", "mix", "comm", "gemm")."""
    want = set(only) if only else {"hip", "mix", "comm", "gemm"}
    LIB.mkdir(exist_ok=True)
    OBJ.mkdir(exist_ok=True)

    # library -> (its sources, its link line); a library newer than its sources and the headers is left alone, object files or not
    # (a checkout that ships built libraries does not ship the objects)
    link = [HIPCC, "-shared", "-fPIC"]
    libs = {
        # --no-undefined: a kernel whose host-side launch stub went missing must fail HERE, not at dlopen on the GPU box
        "hip": (HIP_SOURCES, [*link, f"--offload-arch={ARCH}", "-Wl,--no-undefined"], []),
        "mix": (MIX_SOURCES, [*link, f"--offload-arch={ARCH}", "-Wl,--no-undefined"], []),
        "comm": (COMM_SOURCES, link, ["-L", str(ROCM / "lib"), "-lrccl", f"-Wl,-rpath,{ROCM / 'lib'}"]),
        "gemm": (GEMM_SOURCES, link, ["-L", str(ROCM / "lib"), "-lhipblaslt", f"-Wl,-rpath,{ROCM / 'lib'}"]),
    }
    headers = list(CSRC.glob("*.h")) + list(INCLUDE.glob("*.h"))
    out = {k: LIB / f"libmsgl_{k}.so" for k in libs if k in want}
    todo = {k: [CSRC / n for n in libs[k][0]] for k in out}
    todo = {k: srcs for k, srcs in todo.items() if force or _stale(out[k], srcs + headers)}
    with ThreadPoolExecutor(max_workers=min(16, os.cpu_count() or 1)) as pool:
        objs = {k: [pool.submit(_compile, s, force) for s in srcs] for k, srcs in todo.items()}
        for k, futures in objs.items():
            built = [str(f.result()) for f in futures]
            _run([*libs[k][1], *built, *libs[k][2], "-o", str(out[k])])
    if verbose:
        for k, v in out.items():
            print(f"[build] {k}: {v} ({v.stat().st_size >> 10} KiB)")
    return out


if __name__ == "__main__":
    build_all(force="--force" in sys.argv)
