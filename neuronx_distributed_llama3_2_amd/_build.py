"""In-tree build of the CDNA4 extension `_C` (hipcc --offload-arch=gfx950, no hipify, no JIT cache).

Every `csrc/*.hip` file is a self-contained kernel translation unit (HIP runtime headers only, so
each compiles in seconds); the `csrc/*.cpp` host TUs (pybind bindings, the hipBLASLt GEMM tuner)
are the only ones that include the torch headers.
Objects are cached under `build/` keyed on source + header mtimes and flags and compiled in parallel,
then linked into `_C*.so` and `_hybrid*.so` next to this file, so the built libraries
travel with the source tree (e.g. to a GPU box) and are what `import` loads.

Usage:  python -m neuronx_distributed_llama3_2_amd._build [--force] [--jobs N] [--target _C|_hybrid]
"""

from __future__ import annotations

import argparse
import concurrent.futures as cf
import os
import subprocess
import sys
import sysconfig
from pathlib import Path

PKG_DIR = Path(__file__).resolve().parent
CSRC = PKG_DIR / "csrc"
BUILD_DIR = PKG_DIR.parent / "build" / "nxd_csrc"
ARCH = os.environ.get("NXD_OFFLOAD_ARCH", "gfx950")
EXT_SUFFIX = sysconfig.get_config_var("EXT_SUFFIX") or ".so"
# `_C`: every kernel of csrc/*.hip.  `_hybrid`: the mechanisms of the hybrid decoders
# (csrc/hybrid/: hyper-connections, delta rules, windowed / differential / pooled attention, routed experts) and the
# dense and grouped GEMM dispatch, a small module of its own, so that serving such a model compiles only what it runs.
TARGETS = ("_C", "_hybrid")


def _hipcc() -> str:
    rocm = os.environ.get("ROCM_PATH", "/opt/rocm")
    return os.path.join(rocm, "bin", "hipcc")


def _torch_flags():
    import torch

    tdir = Path(torch.__file__).resolve().parent
    rocm = os.environ.get("ROCM_PATH", "/opt/rocm")
    inc = [
        f"-I{os.path.join(rocm, 'include')}",
        f"-I{tdir / 'include'}",
        f"-I{tdir / 'include' / 'torch' / 'csrc' / 'api' / 'include'}",
        f"-I{sysconfig.get_paths()['include']}",
    ]
    abi = int(torch._C._GLIBCXX_USE_CXX11_ABI)
    defs = [
        "-D__HIP_PLATFORM_AMD__=1",
        "-DUSE_ROCM=1",
        "-DTORCH_EXTENSION_NAME=_C",
        "-DTORCH_API_INCLUDE_EXTENSION_H",
        f"-D_GLIBCXX_USE_CXX11_ABI={abi}",
    ]
    libdir = tdir / "lib"
    libs = [f"-L{libdir}", f"-Wl,-rpath,{libdir}", "-lc10", "-ltorch", "-ltorch_cpu", "-ltorch_python", "-lc10_hip",
            "-ltorch_hip", "-lamdhip64", "-lhipblaslt", "-ldl"]
    return inc, defs, libs


# per-TU extra flags.  flash_attn_bwd: without VGPR-form MFMAs the allocator gives the short S/dP
# chains AGPRs and spills two of the 16 resident dK/dV accumulator tiles to scratch every tile.
_EXTRA_FLAGS = {"flash_attn_bwd": ["-mllvm", "-amdgpu-mfma-vgpr-form"]}


# hipcc -O3 forms packed fp32 instructions (v_pk_{add,mul,fma}_f32) from ordinary float code; some of
# their forms have given wrong results on MI355X now and then, so no device code may contain them
# (the host pass warns that it does not know the feature: harmless).
_NO_PACKED_FP32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _needs_build(src: Path, obj: Path, deps, flags) -> bool:
    """Missing or older than its sources, or compiled with other flags (kept beside the object)."""
    stamp = obj.with_suffix(".flags")
    if not obj.exists() or not stamp.exists() or stamp.read_text() != " ".join(flags):
        return True
    t = obj.stat().st_mtime
    return any(p.stat().st_mtime > t for p in [src, *deps])


def _compile(cmd):
    r = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    return r.returncode, r.stdout, cmd


def _sources(target: str):
    """(kernel TUs, host TUs that include the torch headers) of one extension module."""
    if target == "_C":
        return sorted(CSRC.glob("*.hip")), sorted(CSRC.glob("*.cpp"))
    shared = [CSRC / n for n in ("grouped_gemm.hip", "grouped_rowgemm.hip")]   # the experts' matrix products
    return [*sorted((CSRC / "hybrid").glob("*.hip")), *shared], [*sorted((CSRC / "hybrid").glob("*.cpp")), CSRC / "gemm.cpp"]


def lib_path(target: str) -> Path:
    return PKG_DIR / (target + EXT_SUFFIX)


def build(force: bool = False, jobs: int | None = None, verbose: bool = False, targets=TARGETS) -> Path:
    """Compile and link the extension modules in `targets`; returns the last one's path."""
    hipcc = _hipcc()
    if not os.path.exists(hipcc):
        raise RuntimeError(f"hipcc not found at {hipcc}")
    BUILD_DIR.mkdir(parents=True, exist_ok=True)
    headers = sorted([*CSRC.glob("*.h"), *CSRC.glob("hybrid/*.h")])
    inc, defs, libs = _torch_flags()
    common = ["-O3", "-fPIC", "-std=c++17", f"--offload-arch={ARCH}", "-fno-gpu-rdc", f"-I{CSRC}",
              "-Wno-unused-result", "-Wno-unused-variable", *_NO_PACKED_FP32]
    jobs_list = []
    objs = {}
    stamps = {}
    for target in targets:
        objs[target] = []
        kernels, host = _sources(target)
        for src in [*host, *kernels]:   # the host TUs take longest: start them first
            obj = BUILD_DIR / (src.stem + ".o")
            objs[target].append(obj)
            flags = [*common, *inc, *defs] if src.suffix == ".cpp" else [*common, *_EXTRA_FLAGS.get(src.stem, [])]
            if obj not in stamps and (force or _needs_build(src, obj, headers, flags)):
                lang = ["-x", "hip"] if src.suffix == ".cpp" else []
                jobs_list.append([hipcc, *lang, *flags, "-c", str(src), "-o", str(obj)])
                stamps[obj] = " ".join(flags)
    jobs = jobs or min(8, os.cpu_count() or 4, 16)
    failures = []
    if jobs_list:
        with cf.ThreadPoolExecutor(max_workers=jobs) as ex:
            for rc, out, cmd in ex.map(_compile, jobs_list):
                if verbose or rc != 0:
                    sys.stderr.write(out)
                obj = Path(cmd[-1])
                if rc != 0:
                    failures.append(" ".join(cmd))
                else:
                    obj.with_suffix(".flags").write_text(stamps[obj])
    if failures:
        raise RuntimeError("HIP compilation failed:\n" + "\n".join(failures))
    path = None
    for target in targets:
        path = lib_path(target)
        if force or not path.exists() or any(o in stamps or o.stat().st_mtime > path.stat().st_mtime
                                             for o in objs[target]):
            tmp = path.with_suffix(".tmp.so")
            cmd = [hipcc, "-shared", "-fPIC", f"--offload-arch={ARCH}", "-fno-gpu-rdc", *map(str, objs[target]), "-o",
                   str(tmp), *libs]
            rc, out, _ = _compile(cmd)
            if rc != 0:
                sys.stderr.write(out)
                raise RuntimeError("link failed: " + " ".join(cmd))
            os.replace(tmp, path)
    return path


def main(argv=None):
    ap = argparse.ArgumentParser()
    ap.add_argument("--force", action="store_true")
    ap.add_argument("--jobs", type=int, default=None)
    ap.add_argument("--verbose", action="store_true")
    ap.add_argument("--target", action="append", choices=TARGETS, default=None, help="default: all modules")
    a = ap.parse_args(argv)
    p = build(force=a.force, jobs=a.jobs, verbose=a.verbose, targets=tuple(a.target or TARGETS))
    print(p)


if __name__ == "__main__":
    main()
