"""Native build driver: HIP kernels (gfx950) and the C++ host runtime.

Everything is compiled in-tree into ``cake_amd/lib/`` so the shared objects
travel with the repository snapshot to the GPU box:

* ``libcake_gemm.so`` (``csrc/kernels/gemm*.hip``), ``libcake_mixers.so``
  (``csrc/kernels/mixer_*.hip``: the hybrid designs' layers) and
  ``libcake_kernels.so`` (every other ``csrc/kernels/*.hip`` file), ``hipcc
  --offload-arch=gfx950``; plain C ABI (``extern "C" cake_*``) driven from
  :mod:`cake_amd.ops` through ctypes with torch's current HIP stream, so
  the launches are capturable in hipGraphs.  ``libcake_kernels.so`` needs
  ``libcake_gemm.so`` and also holds ``csrc/driver/*.cpp``: the
  native decode loop that replays the captured step graphs
  (:mod:`cake_amd.ops.graph_loop`).  The split lets a program that serves one
  model compile only what that model runs (:func:`ensure_text`).
* ``libcake_runtime.so`` — ``csrc/runtime/*.cpp`` (topology parser, wire codec,
  safetensors mmap reader/writer, framed TCP transport), C ABI.
* ``cake-split-model`` — native executable (``csrc/tools/split_model.cpp``).
* ``cake-cli`` — the native entry point (``csrc/tools/cake_cli.cpp``): flags,
  validation and topology natively, compute runtime embedded in-process
  (libpython); ``libcake_runtime.so``'s ``cake_start_worker`` embeds the same way.

Object files are cached under ``build/`` keyed on mtimes of the source and the
shared headers, so re-running is cheap.

Usage: ``python -m cake_amd.build [--force] [-j N]``
"""
from __future__ import annotations

import argparse
import concurrent.futures as cf
import os
import shutil
import subprocess
import sys
from pathlib import Path

PKG = Path(__file__).resolve().parent
CSRC = PKG / "csrc"
LIB = PKG / "lib"
BUILD = PKG.parent / "build" / "native"
ARCH = os.environ.get("CAKE_OFFLOAD_ARCH", "gfx950")

HIPCC = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
CXX = shutil.which("g++") or "c++"

KERNEL_LIB = LIB / "libcake_kernels.so"
GEMM_LIB = LIB / "libcake_gemm.so"
MIXER_LIB = LIB / "libcake_mixers.so"
RUNTIME_LIB = LIB / "libcake_runtime.so"
SPLIT_TOOL = LIB / "cake-split-model"
CLI_TOOL = LIB / "cake-cli"


def _newer(src: Path, deps: list[Path], out: Path) -> bool:
    if not out.exists():
        return True
    t = out.stat().st_mtime
    return any(p.stat().st_mtime > t for p in [src, *deps] if p.exists())


def _run(cmd: list[str]) -> None:
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"command failed ({r.returncode}): {' '.join(cmd)}\n{r.stdout}\n{r.stderr}")


# packed FP32 math stays off in every HIP object: some v_pk_*_f32 forms the compiler picks by
# itself have given wrong results now and then on this hardware, with no error
# per-file hipcc flags: the GEMM's compile-time-unrolled interleaved schedule needs its
# lambdas fully inlined (below the default threshold the 128x128-per-wave tile keeps
# closures in scratch memory)
NO_PK_FP32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
HIP_EXTRA = {"gemm": ["-mllvm", "-inline-threshold=100000"]}  # gemm.hip and gemm_inst_*.hip


def _compile_hip(src: Path, force: bool) -> Path:
    out = BUILD / "kernels" / (src.stem + ".o")
    out.parent.mkdir(parents=True, exist_ok=True)
    headers = sorted((CSRC / "kernels").glob("*.h"))
    if force or _newer(src, headers, out):
        _run([HIPCC, "-O3", f"--offload-arch={ARCH}", "-std=c++17", "-fPIC",
              "-Wno-unused-result", "-munsafe-fp-atomics", *NO_PK_FP32,
              *HIP_EXTRA.get(src.stem.split("_")[0], []),
              "-c", str(src), "-o", str(out)])
    return out


def _compile_cpp(src: Path, force: bool, extra: list[str] | None = None) -> Path:
    out = BUILD / "runtime" / (src.stem + ".o")
    out.parent.mkdir(parents=True, exist_ok=True)
    headers = sorted((CSRC / "runtime").glob("*.h")) + [CSRC / "engine" / "llama_engine.h"]
    if force or _newer(src, headers, out):
        _run([CXX, "-O2", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function",
              "-fvisibility=hidden", *(extra or []), "-c", str(src), "-o", str(out)])
    return out


def _py_ext_flags() -> tuple[list[str], str]:
    import sysconfig

    import pybind11
    inc = [f"-I{pybind11.get_include()}", f"-I{sysconfig.get_paths()['include']}"]
    return inc, sysconfig.get_config_var("EXT_SUFFIX") or ".so"


PY_EXT = LIB / "_cake_runtime"  # + EXT_SUFFIX

EXPERIMENTAL = os.environ.get("CAKE_BUILD_EXPERIMENTAL", "0") != "0"


def _kernel_sources() -> dict[Path, list[Path]]:
    """Shared object -> its sources.  csrc/experimental (the persistent decode engine,
    measured slower than the launch path: profiles/r4_mk_summary.md) only with
    CAKE_BUILD_EXPERIMENTAL=1."""
    hip = sorted((CSRC / "kernels").glob("*.hip"))
    gemm = [p for p in hip if p.stem == "gemm" or p.stem.startswith("gemm_inst")]
    mixers = [p for p in hip if p.stem.startswith("mixer_")]
    rest = [p for p in hip if p not in gemm and p not in mixers]
    rest += sorted((CSRC / "driver").glob("*.cpp"))
    if EXPERIMENTAL:
        rest += sorted((CSRC / "experimental").glob("*.hip"))
    return {GEMM_LIB: gemm, MIXER_LIB: mixers, KERNEL_LIB: rest}


def build_kernels(force: bool = False, jobs: int = 8,
                  libs: tuple[Path, ...] = (GEMM_LIB, MIXER_LIB, KERNEL_LIB)) -> Path:
    # HIP kernels + the native graph-replay decode driver (host code on the HIP runtime)
    groups = {lib: srcs for lib, srcs in _kernel_sources().items() if lib in libs}
    # the GEMM instantiations compile longest: first in the queue
    todo = sorted((s for srcs in groups.values() for s in srcs),
                  key=lambda p: not p.stem.startswith("gemm_inst"))
    with cf.ThreadPoolExecutor(max_workers=jobs) as ex:
        objs = dict(zip(todo, ex.map(lambda s: _compile_hip(s, force), todo)))
    LIB.mkdir(parents=True, exist_ok=True)
    keep = {BUILD / "kernels" / (s.stem + ".o")
            for srcs in _kernel_sources().values() for s in srcs}
    stale = [o for o in (BUILD / "kernels").glob("*.o") if o not in keep]
    for o in stale:  # an object of a source no longer built (experimental off) must go
        o.unlink()
    for lib, srcs in groups.items():
        mine = [objs[s] for s in srcs]
        # hipBLASLt for the plain prefill GEMMs it measured faster on (driver/blaslt.cpp);
        # in a torch process the soname resolves to the copy torch already loaded
        extra = [] if lib != KERNEL_LIB else [
            "-L/opt/rocm/lib", "-lhipblaslt", f"-L{LIB}", "-Wl,--no-as-needed", "-lcake_gemm",
            "-Wl,-rpath,$ORIGIN"]
        if force or stale or any(_newer(o, [], lib) for o in mine):
            # --no-undefined: a kernel whose host stub the compiler dropped fails here, not at
            # dlopen on the GPU box
            tmp = lib.with_suffix(f".tmp{os.getpid()}")
            _run([HIPCC, f"--offload-arch={ARCH}", "-shared", "-fPIC", *map(str, mine),
                  "-o", str(tmp), f"-Wl,-soname,{lib.name}", *extra, "-Wl,--no-undefined"])
            os.replace(tmp, lib)
    return KERNEL_LIB


def _embed_flags() -> tuple[list[str], list[str]]:
    """Compile / link flags to embed libpython (python3-config --embed equivalent)."""
    import sysconfig
    inc = [f"-I{sysconfig.get_paths()['include']}"]
    ver = sysconfig.get_config_var("LDVERSION") or sysconfig.get_python_version()
    libdir = sysconfig.get_config_var("LIBDIR") or "/usr/lib"
    return inc, [f"-L{libdir}", f"-lpython{ver}", "-ldl", "-lm", "-lpthread"]


def build_runtime_module(force: bool = False, jobs: int = 8) -> tuple[Path, list[Path]]:
    """The pybind11 module of the C++ host runtime (safetensors reader, topology, codec)."""
    rt = CSRC / "runtime"
    core_srcs = [rt / f"{n}.cpp" for n in ("json", "topology", "proto", "net", "safetensors",
                                            "server", "native_worker")]
    inc, ext = _py_ext_flags()
    with cf.ThreadPoolExecutor(max_workers=jobs) as ex:
        bind_f = ex.submit(_compile_cpp, rt / "bindings.cpp", force, inc)
        core = list(ex.map(lambda s: _compile_cpp(s, force), core_srcs))
        bind = bind_f.result()
    LIB.mkdir(parents=True, exist_ok=True)
    pyext = PY_EXT.with_name(PY_EXT.name + ext)
    if force or any(_newer(o, [], pyext) for o in [*core, bind]):
        _run([CXX, "-shared", "-fPIC", *map(str, core), str(bind), "-o", str(pyext), "-lpthread",
              "-ldl"])
    return pyext, core


def build_runtime(force: bool = False, jobs: int = 8) -> Path:
    """C++ host runtime: pybind11 module, C-ABI library, split-model tool and cake-cli."""
    rt = CSRC / "runtime"
    einc, elink = _embed_flags()
    pyext, core = build_runtime_module(force, jobs)
    with cf.ThreadPoolExecutor(max_workers=jobs) as ex:
        capi_f = ex.submit(_compile_cpp, rt / "capi.cpp", force)
        emb_f = ex.submit(_compile_cpp, rt / "embed.cpp", force, einc)
        capi, emb = capi_f.result(), emb_f.result()
    if force or any(_newer(o, [], RUNTIME_LIB) for o in [*core, capi, emb]):
        _run([CXX, "-shared", "-fPIC", *map(str, core), str(capi), str(emb), "-o",
              str(RUNTIME_LIB), *elink])
    tool = CSRC / "tools" / "split_model.cpp"
    if force or _newer(tool, [*core, *sorted(rt.glob("*.h"))], SPLIT_TOOL):
        _run([CXX, "-O2", "-std=c++17", f"-I{rt}", str(tool), *map(str, core), "-o",
              str(SPLIT_TOOL), "-lpthread", "-ldl"])
    cli = CSRC / "tools" / "cake_cli.cpp"
    if force or _newer(cli, [*core, emb, *sorted(rt.glob("*.h")), CSRC / "engine" / "llama_engine.h"],
                       CLI_TOOL):
        _run([CXX, "-O2", "-std=c++17", f"-I{rt}", str(cli), *map(str, core), str(emb), "-o",
              str(CLI_TOOL), *elink])
    return pyext


ENGINE_LIB = LIB / "libcake_engine.so"


def build_engine(force: bool = False) -> Path:
    """Native engines (csrc/engine: Llama, Stable Diffusion): host C++ on the HIP runtime
    over the kernel library's C entry points, plus the runtime's JSON / safetensors
    readers."""
    rt = CSRC / "runtime"
    objs = [_compile_cpp(rt / f"{n}.cpp", force) for n in ("json", "safetensors", "net", "proto")]
    deps = [*sorted((CSRC / "engine").glob("*.h")), *sorted(rt.glob("*.h")),
            CSRC / "driver" / "graph_loop.h"]
    eng_objs = []
    for src in sorted((CSRC / "engine").glob("*.cpp")):  # llama_engine, sd_engine
        out = BUILD / "engine" / (src.stem + ".o")
        out.parent.mkdir(parents=True, exist_ok=True)
        if force or _newer(src, deps, out):
            _run([HIPCC, "-O2", "-std=c++17", "-fPIC", "-fvisibility=hidden", "-Wall",
                  "-Wno-unused-function", "-c", str(src), "-o", str(out)])
        eng_objs.append(out)
    if force or any(_newer(o, [], ENGINE_LIB) for o in [*eng_objs, *objs, KERNEL_LIB]):
        _run([HIPCC, "-shared", "-fPIC", *map(str, eng_objs), *map(str, objs), "-o",
              str(ENGINE_LIB), f"-L{LIB}", "-lcake_kernels", "-lcake_gemm", "-Wl,-rpath,$ORIGIN",
              "-Wl,--no-undefined"])
    return ENGINE_LIB


def ensure_text(libs: tuple[str, ...], jobs: int | None = None) -> None:
    """Compile what is missing for a text model run from this checkout: the named kernel
    libraries ("gemm", "mixers", "kernels") and the runtime module.  Libraries that are
    there already are used as they are."""
    jobs = jobs or int(os.environ.get("MAX_JOBS") or min(16, os.cpu_count() or 4))
    paths = {"gemm": GEMM_LIB, "mixers": MIXER_LIB, "kernels": KERNEL_LIB}
    need = tuple(paths[n] for n in libs if not paths[n].exists())
    if KERNEL_LIB in need and not GEMM_LIB.exists() and GEMM_LIB not in need:
        need = (GEMM_LIB, *need)
    if not PY_EXT.with_name(PY_EXT.name + _py_ext_flags()[1]).exists():
        build_runtime_module(jobs=jobs)
    if need:
        build_kernels(jobs=jobs, libs=need)


def build_all(force: bool = False, jobs: int = 8) -> None:
    build_kernels(force, jobs)
    build_engine(force)
    build_runtime(force, jobs)


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(description=__doc__.splitlines()[0])
    ap.add_argument("--force", action="store_true")
    ap.add_argument("-j", "--jobs", type=int, default=min(8, os.cpu_count() or 4))
    ap.add_argument("--only", choices=["kernels", "engine", "runtime"], default=None)
    a = ap.parse_args(argv)
    if a.only in (None, "kernels"):
        print("built", build_kernels(a.force, a.jobs))
    if a.only in (None, "engine"):
        print("built", build_engine(a.force))
    if a.only in (None, "runtime"):
        print("built", build_runtime(a.force, a.jobs))
    return 0


if __name__ == "__main__":
    sys.exit(main())
