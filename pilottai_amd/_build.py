"""In-tree builder for the native parts of pilottai_amd.

Five shared objects are produced next to the Python sources so they travel with
the repository snapshot to the GPU box:

* ``pilottai_amd/_C.so``       — CDNA4 HIP kernels (csrc/ops/*.hip, gfx950 only)
                                  + torch/pybind11 bindings (csrc/ops/bindings.cpp)
* ``pilottai_amd/_latent.so`` — the kernels of models with latent attention and table-routed
                                  experts, with the packed projections they share (so that
                                  such a model needs no other kernel to run)
* ``pilottai_amd/_hybrid.so`` — likewise for models with paged attention of many kinds, recurrent layers,
                                  score-routed experts and fp32 residuals
* ``pilottai_amd/_latent_linear.so`` — likewise for models that mix latent attention with gated linear attention
* ``pilottai_amd/_runtime.so`` — C++ serving runtime: paged-KV block manager,
                                  prefix cache, continuous-batching scheduler,
                                  grammar FSM + tokenizer (csrc/runtime/*.cpp),
                                  pybind11 bindings, no GPU code.

hipcc is driven directly (no hipify, no torch JIT cache): each translation unit
is compiled to an object in ``build/`` and re-linked only when a source or
header changed. Usage: ``python -m pilottai_amd._build`` or ``build_all()``.
"""
from __future__ import annotations

import concurrent.futures as cf
import glob
import os
import subprocess
import sys
import sysconfig
from pathlib import Path

ROOT = Path(__file__).resolve().parent.parent
PKG = ROOT / "pilottai_amd"
CSRC = ROOT / "csrc"
BUILD = ROOT / "build"
ARCH = os.environ.get("PILOTTAI_GPU_ARCH", "gfx950")
HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
# Per-file code-generation flags. gemm_mid.hip: MFMA accumulators in the VGPR form; with
# the AGPR form hipcc shuffles them through v_accvgpr moves in the software-pipelined loop.
# No file may use packed fp32 arithmetic (v_pk_*_f32): some forms have given wrong results.
HIP_FLAGS = ["-ffast-math", "-fno-gpu-rdc", "-Wno-unused-result", "-Xclang", "-target-feature", "-Xclang",
             "-packed-fp32-ops"]
# kernel modules of the families beside Llama: sources and bindings; the GEMM sources are in _C.so too
SHARED_HIP = ["gemm_decode.hip", "gemm_prefill.hip"]
MODULES = {
    "latent": (["grouped_gemm.hip", "latent_attention.hip", "latent_cache.hip", "residual_norm.hip"], "bindings_latent.cpp"),
    "hybrid": (["gated_norm.hip", "grouped_gemm.hip", "head_difference.hip", "hyper_norm.hip", "matrix_memory.hip", "paged_kv.hip",
                "score_route.hip", "state_scan.hip", "window_attention.hip"], "bindings_hybrid.cpp"),
    "latent_linear": (["gated_norm.hip", "grouped_gemm.hip", "latent_attention.hip", "latent_cache.hip", "linear_attention.hip",
                       "poly_norm.hip", "residual_norm.hip", "score_route.hip"], "bindings_latent_linear.cpp"),
}
FAMILY_HIP = {h for hips, _ in MODULES.values() for h in hips}
FILE_FLAGS = {"gemm_mid.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form"],
              "gemm_stream.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form"]}


def _torch_paths():
    from torch.utils import cpp_extension as ce

    return ce.include_paths(), ce.library_paths()


def _py_include() -> str:
    return sysconfig.get_paths()["include"]


def _pybind_include() -> str:
    import pybind11

    return pybind11.get_include()


def _newest(paths) -> float:
    return max((os.path.getmtime(p) for p in paths), default=0.0)


def _run(cmd):
    r = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    if r.returncode != 0:
        raise RuntimeError("command failed:\n" + " ".join(cmd) + "\n" + r.stdout)
    return r.stdout


_FORCE = False  # compile up-to-date objects too


def _compile_many(jobs, workers: int):
    todo = [(src, obj, cmd) for src, obj, cmd, deps in jobs
            if _FORCE or not os.path.exists(obj) or os.path.getmtime(obj) < _newest([src] + deps)]
    if not todo:
        return 0
    with cf.ThreadPoolExecutor(max_workers=max(1, workers)) as ex:
        futs = [ex.submit(_run, cmd) for _, _, cmd in todo]
        for f in futs:
            f.result()
    return len(todo)


def _build_ext(name: str, hips, binding: str, verbose: bool, workers: int | None) -> Path:
    """Compile csrc/ops sources and one binding file into pilottai_amd/<name>.so (gfx950 code objects)."""
    incs, libdirs = _torch_paths()
    out = PKG / (name + sysconfig.get_config_var("EXT_SUFFIX"))
    BUILD.mkdir(exist_ok=True)
    headers = glob.glob(str(CSRC / "ops" / "*.h"))
    jobs = []
    objs = []
    for src in hips:
        src = str(CSRC / "ops" / src)
        obj = str(BUILD / (Path(src).stem + ".hip.o"))
        cmd = [HIPCC, f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC", "-c", src,
               "-o", obj, *HIP_FLAGS, *FILE_FLAGS.get(Path(src).name, [])]
        jobs.append((src, obj, cmd, headers))
        objs.append(obj)
    bsrc = str(CSRC / "ops" / binding)
    bobj = str(BUILD / f"ops_{Path(binding).stem}.o")
    defs = ["-D__HIP_PLATFORM_AMD__=1", "-DUSE_ROCM=1", f"-DTORCH_EXTENSION_NAME={name}",
            "-DTORCH_API_INCLUDE_EXTENSION_H", "-D_GLIBCXX_USE_CXX11_ABI=1"]
    bcmd = ["g++", "-O2", "-std=c++17", "-fPIC", "-c", bsrc, "-o", bobj, *defs,
            "-I/opt/rocm/include", f"-I{_py_include()}"] + [f"-I{i}" for i in incs]
    jobs.append((bsrc, bobj, bcmd, headers))
    objs.append(bobj)
    n = _compile_many(jobs, workers or min(8, os.cpu_count() or 4))
    if n or not out.exists() or out.stat().st_mtime < _newest(objs):
        part = str(out) + f".{os.getpid()}"  # several processes may build at once: rename into place
        link = [HIPCC, "-shared", "-fPIC", f"--offload-arch={ARCH}", "-o", part, *objs]
        for d in libdirs:
            link += [f"-L{d}", f"-Wl,-rpath,{d}"]
        link += ["-lc10", "-lc10_hip", "-ltorch", "-ltorch_cpu", "-ltorch_hip",
                 "-ltorch_python", "-lamdhip64"]
        _run(link)
        os.replace(part, out)
        if verbose:
            print(f"[pilottai_amd] linked {out}")
    return out


def build_ops(verbose: bool = False, workers: int | None = None) -> Path:
    """pilottai_amd/_C.so: every kernel but the other families' own."""
    hips = sorted(Path(p).name for p in glob.glob(str(CSRC / "ops" / "*.hip")))
    return _build_ext("_C", [h for h in hips if h not in FAMILY_HIP], "bindings.cpp", verbose, workers)


def build_family(kind: str, verbose: bool = False, workers: int | None = None) -> Path:
    """pilottai_amd/_<kind>.so: what a model of that family runs."""
    hips, binding = MODULES[kind]
    return _build_ext("_" + kind, hips + SHARED_HIP, binding, verbose, workers)


def build_runtime(verbose: bool = False, workers: int | None = None) -> Path:
    """Compile csrc/runtime (pure C++17, no torch) into pilottai_amd/_runtime.so."""
    out = PKG / ("_runtime" + sysconfig.get_config_var("EXT_SUFFIX"))
    BUILD.mkdir(exist_ok=True)
    srcs = sorted(glob.glob(str(CSRC / "runtime" / "*.cpp")))
    headers = glob.glob(str(CSRC / "runtime" / "*.h"))
    jobs, objs = [], []
    flags = os.environ.get("PILOTTAI_RUNTIME_CXXFLAGS", "-O3").split()
    for src in srcs:
        obj = str(BUILD / (Path(src).stem + ".rt.o"))
        cmd = ["g++", *flags, "-std=c++17", "-fPIC", "-Wall", "-c", src, "-o", obj,
               f"-I{_py_include()}", f"-I{_pybind_include()}", f"-I{CSRC / 'runtime'}"]
        jobs.append((src, obj, cmd, headers))
        objs.append(obj)
    n = _compile_many(jobs, workers or min(8, os.cpu_count() or 4))
    if objs and (n or not out.exists() or out.stat().st_mtime < _newest(objs)):
        _run(["g++", "-shared", "-fPIC", *flags, "-o", str(out), *objs, "-lpthread"])
        if verbose:
            print(f"[pilottai_amd] linked {out}")
    return out


def _stale(so: Path, sources) -> bool:
    return not so.exists() or so.stat().st_mtime < _newest(sources)


def ensure(kind: str, gpu: bool = True) -> None:
    """Build what running a model of `kind` needs, where it is missing or older than its sources: the
    serving runtime and, for a GPU, the kernel module (one of MODULES, or _C for "llama"). One process
    builds at a time; the others wait for it."""
    import fcntl

    ext = sysconfig.get_config_var("EXT_SUFFIX")
    ops_dir = CSRC / "ops"
    srcs = [str(p) for p in ops_dir.glob("*.h")]
    if kind in MODULES:
        hips, binding = MODULES[kind]
        name, srcs = "_" + kind, srcs + [str(ops_dir / h) for h in hips + SHARED_HIP + [binding]]
    else:
        name = "_C"
        srcs += [str(p) for p in ops_dir.glob("*.hip") if p.name not in FAMILY_HIP] + [str(ops_dir / "bindings.cpp")]
    rt = [str(p) for p in (CSRC / "runtime").glob("*.*")]
    build_kernels = (lambda: build_family(kind)) if kind in MODULES else build_ops

    def todo():
        return [f for f, so, src in ((build_runtime, PKG / ("_runtime" + ext), rt), (build_kernels, PKG / (name + ext), srcs))
                if _stale(so, src) and (gpu or f is build_runtime)]

    if not todo():
        return
    BUILD.mkdir(exist_ok=True)
    with open(BUILD / ".lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        for f in todo():
            f()


def build_all(verbose: bool = False, force: bool = False) -> None:
    global _FORCE
    _FORCE = force
    try:
        build_runtime(verbose)
        for kind in MODULES:
            build_family(kind, verbose)
        build_ops(verbose)
    finally:
        _FORCE = False


if __name__ == "__main__":
    build_all(verbose=True)
    sys.exit(0)
