#!/usr/bin/env python3
"""Build the native (HIP/C++) parts of kvmini in-tree for gfx950.

* ``kvmini/_C.<abi>.so``       torch extension: HIP kernels (csrc/*.hip) + bindings.cpp
* ``kvmini/libkvmini_rt.so``      torch-free amd-smi sampler thread, loaded through ctypes
* ``kvmini/libkvmini_gather.so``  RCCL telemetry all-gather (binds to the process's HIP/RCCL at load)

hipcc cross-compiles for gfx950 without a GPU, so this runs on a CPU-only build
host; objects are cached under ``build/`` by source mtime.  ``python build_native.py``
builds everything, ``--force`` rebuilds, ``--only ext|rt`` picks one target.
"""

from __future__ import annotations

import argparse
import concurrent.futures
import os
import shlex
import subprocess
import sys
import sysconfig
from pathlib import Path

ROOT = Path(__file__).resolve().parent
CSRC = ROOT / "csrc"
BUILD = ROOT / "build"
ARCH = os.environ.get("KVMINI_GPU_ARCH", "gfx950")
HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
CXX = os.environ.get("CXX", "g++")
ROCM = os.environ.get("ROCM_PATH", "/opt/rocm")

# Packed fp32 instructions (two fp32 operations per lane, which the optimiser forms on its own from scalar code) have
# given wrong results on gfx950 in some of their forms: no device code is compiled with them.
DEVICE_FLAGS = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

KERNEL_SOURCES = ["hist_quantile.hip", "energy_trapz.hip", "engine_kernels.hip", "stream_gemm.hip", "wide_gemm.hip", "mfma_scaled.hip", "sampling.hip", "guided.hip", "xgmi_collectives.hip",
                  "mixer_kernels.hip", "chunk_attention.hip", "delta_rule.hip", "latent_attention.hip", "retention.hip", "state_space.hip", "experts.hip"]
BINDING_SOURCES = ["bindings.cpp", "mixer_bindings.cpp"]


def run(cmd: list[str]) -> None:
    print("+", " ".join(shlex.quote(c) for c in cmd), flush=True)
    subprocess.run(cmd, check=True)


def stale(out: Path, deps: list[Path]) -> bool:
    if not out.exists():
        return True
    t = out.stat().st_mtime
    return any(d.stat().st_mtime > t for d in deps)


def ext_path() -> Path:
    return ROOT / "kvmini" / ("_C" + sysconfig.get_config_var("EXT_SUFFIX"))


def compile_all(jobs: list[tuple[Path, Path, list[str]]], force: bool) -> list[Path]:
    """Compile (source, object, command) entries whose object is missing, older than its source or was made by another
    command line; several at a time (``MAX_JOBS``, else the CPUs), the largest sources first."""
    todo = []
    for src, obj, cmd in jobs:
        note = obj.with_suffix(".cmd")
        if force or stale(obj, [src, *CSRC.glob("*.h")]) or not note.exists() or note.read_text() != shlex.join(cmd):
            todo.append((src, obj, cmd, note))
    todo.sort(key=lambda j: -j[0].stat().st_size)

    def one(job: tuple[Path, Path, list[str], Path]) -> None:
        _src, obj, cmd, note = job
        part = obj.with_suffix(f".{os.getpid()}.part")
        run([*cmd, "-o", str(part)])
        part.replace(obj)
        note.write_text(shlex.join(cmd))

    if todo:
        with concurrent.futures.ThreadPoolExecutor(int(os.environ.get("MAX_JOBS", "0")) or min(16, os.cpu_count() or 4)) as pool:
            for f in [pool.submit(one, j) for j in todo]:
                f.result()
    return [obj for _src, obj, _cmd in jobs]


def build_ext(force: bool = False) -> Path:
    import torch
    from torch.utils import cpp_extension as ce

    BUILD.mkdir(exist_ok=True)
    device = [HIPCC, f"--offload-arch={ARCH}", *DEVICE_FLAGS]
    jobs = [(CSRC / src, BUILD / (Path(src).stem + ".o"), [*device, "-O3", "-std=c++17", "-fPIC", "-c", str(CSRC / src)]) for src in KERNEL_SOURCES]
    # bindings: torch headers (slow to parse) — compiled as HIP so the HIP runtime types resolve
    inc = []
    for p in ce.include_paths():
        inc += ["-isystem", p]
    inc += ["-isystem", sysconfig.get_paths()["include"]]
    for src in BINDING_SOURCES:
        jobs.append((CSRC / src, BUILD / (Path(src).stem + ".o"),
                     [*device, "-x", "hip", "-O2", "-std=c++17", "-fPIC", "-D__HIP_PLATFORM_AMD__=1", "-DUSE_ROCM=1", "-DHIPBLAS_V2",
                      f"-D_GLIBCXX_USE_CXX11_ABI={int(torch._C._GLIBCXX_USE_CXX11_ABI)}", "-DTORCH_EXTENSION_NAME=_C", "-DTORCH_API_INCLUDE_EXTENSION_H",
                      "-Wno-deprecated-declarations", *inc, "-c", str(CSRC / src)]))
    objs = compile_all(jobs, force)
    out = ext_path()
    if force or stale(out, objs):
        libdirs = ce.library_paths()
        link = []
        for d in libdirs:
            link += [f"-L{d}", f"-Wl,-rpath,{d}"]
        # linked with the host C++ driver, not hipcc: hipcc would add the SYSTEM libamdhip64 next
        # to the one bundled with torch, and a process with two HIP runtimes fails in odd ways
        # (kernel launches of the second one report "no ROCm-capable device")
        run([CXX, "-shared", "-fPIC", *map(str, objs), *link, "-lc10", "-lc10_hip", "-ltorch_cpu", "-ltorch_hip", "-ltorch", "-ltorch_python", "-lamdhip64", "-o", str(out)])
    return out


def rt_path() -> Path:
    return ROOT / "kvmini" / "libkvmini_rt.so"


def gather_path() -> Path:
    return ROOT / "kvmini" / "libkvmini_gather.so"


def build_rt(force: bool = False) -> Path:
    """Two torch-free libraries.  ``libkvmini_rt.so`` (amd-smi sampler thread, which opens
    libamd_smi with dlopen, and the analysis host routines) links no GPU runtime at all, so it can be loaded into any process
    at any time.  ``libkvmini_gather.so`` (RCCL telemetry all-gather) uses HIP + RCCL but is
    linked WITHOUT them: its loader (kvmini/telemetry/native_rt.py) first makes the process's
    one HIP runtime and RCCL global — the copies bundled with torch when torch is imported,
    the system ones otherwise — so a process never ends up with two HIP runtimes."""
    BUILD.mkdir(exist_ok=True)
    out = rt_path()
    srcs = [s for s in (CSRC / "amdsmi_sampler.cpp", CSRC / "host_routines.cpp") if s.exists()]
    if srcs and (force or stale(out, srcs)):
        run([CXX, "-O2", "-std=c++17", "-fPIC", "-shared", *map(str, srcs), "-lpthread", "-ldl", "-o", str(out)])
    gout = gather_path()
    gsrc = CSRC / "telemetry_gather.cpp"
    if gsrc.exists() and (force or stale(gout, [gsrc])):
        run([CXX, "-O2", "-std=c++17", "-fPIC", "-shared", "-D__HIP_PLATFORM_AMD__=1", f"-I{ROCM}/include", str(gsrc), "-lpthread", "-o", str(gout)])
    return out


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--force", action="store_true")
    ap.add_argument("--only", choices=["ext", "rt"], default=None)
    a = ap.parse_args()
    if a.only in (None, "ext"):
        print("built", build_ext(a.force))
    if a.only in (None, "rt"):
        print("built", build_rt(a.force))
    return 0


if __name__ == "__main__":
    sys.exit(main())
