"""Native build driver (no setuptools/hipify involved).

* ``_vwa_kernels.so`` -- the gfx950 HIP kernel library + torch bindings. Every ``csrc/kernels/*.hip``
  is compiled with ``hipcc --offload-arch=gfx950`` into its own object (parallel, incremental),
  ``csrc/bindings.cpp`` is compiled against the torch headers, and the lot is linked against
  torch's own HIP runtime (same ``libamdhip64.so.7`` soname, so one HIP runtime per process).
* ``_vwa_core.so`` -- the same bindings over the kernels of CORE only (GEMMs, elementwise, sampling,
  windowed and latent attention, recurrences, routed experts); the launchers of the other files are stubs that fail with a code
  (csrc/core_stubs.cpp).  The command-line entry points build it when a checkout has no library at
  all and the model at hand runs no chained launch: seconds instead of the minutes chain.hip takes.
* ``_vwa_native.so`` -- the CPU runtime library (grammar engine, KV block manager): plain C++17
  with pybind11, built with g++.

Both land in-tree next to this file so they travel with the repo snapshot to the GPU box.
Run: ``python -m voice_enabled_browser_automation_amd.ops.build [--force]``.
"""
from __future__ import annotations

import concurrent.futures as cf
import contextlib
import glob
import os
import re
import subprocess
import sys
import sysconfig

HERE = os.path.dirname(os.path.abspath(__file__))
REPO = os.path.dirname(os.path.dirname(HERE))
CSRC = os.path.join(REPO, "csrc")
BUILD = os.path.join(REPO, "build", "native")
ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950")
HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")

KERNEL_SO = os.path.join(HERE, "_vwa_kernels.so")
CORE_SO = os.path.join(HERE, "_vwa_core.so")
NATIVE_SO = os.path.join(HERE, "_vwa_native.so")


def _torch_paths():
    import torch

    root = os.path.dirname(torch.__file__)
    inc = [os.path.join(root, "include"), os.path.join(root, "include", "torch", "csrc", "api", "include")]
    lib = os.path.join(root, "lib")
    abi = int(torch._C._GLIBCXX_USE_CXX11_ABI)
    return inc, lib, abi


def _py_include():
    return sysconfig.get_paths()["include"]


def _pybind_include():
    import pybind11

    return pybind11.get_include()


def _newer(target: str, deps: list[str]) -> bool:
    if not os.path.exists(target):
        return False
    t = os.path.getmtime(target)
    return all(os.path.getmtime(d) <= t for d in deps)


def _deps(src: str) -> list[str]:
    """The source and every header of this tree it includes, directly or through another."""
    seen, todo = [], [src]
    while todo:
        p = todo.pop()
        if p in seen or not os.path.exists(p):
            continue
        seen.append(p)
        with open(p, encoding="utf-8") as fh:
            for inc in re.findall(r'^\s*#include\s+"([^"]+)"', fh.read(), re.M):
                todo += [os.path.join(os.path.dirname(p), inc), os.path.join(CSRC, inc)]
    return seen


def _run(cmd: list[str]) -> None:
    r = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    if r.returncode != 0:
        sys.stderr.write(r.stdout)
        raise RuntimeError("build step failed: " + " ".join(cmd[:6]) + " ...")


# kernel files the core library holds; launchers of the others are stubs there
CORE = ("gemm", "gemm_f32", "skinny_stream", "elementwise", "stack_ops", "talk_attention", "recurrence", "rglru", "latent", "latent_prefill", "moe",
        "sample")


def build_kernels(force: bool = False, jobs: int = 8, core: bool = False) -> str:
    with _build_lock():
        return _build_kernels(force, jobs, core)


@contextlib.contextmanager
def _build_lock():
    """One builder per checkout at a time (two processes would write the same objects)."""
    import fcntl

    os.makedirs(BUILD, exist_ok=True)
    with open(os.path.join(BUILD, ".lock"), "w") as fh:
        fcntl.flock(fh, fcntl.LOCK_EX)
        yield


def _build_kernels(force: bool, jobs: int, core: bool) -> str:
    inc, lib, abi = _torch_paths()
    kern_src = sorted(glob.glob(os.path.join(CSRC, "kernels", "*.hip")))
    if core:
        kern_src = [s for s in kern_src if os.path.splitext(os.path.basename(s))[0] in CORE]
    target = CORE_SO if core else KERNEL_SO
    # packed f32 arithmetic stays off: some of its forms have given wrong results on these GPUs
    common = [HIPCC, f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC", "-Wno-unused-result",
              "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops", "-I", os.path.join(CSRC)] + os.environ.get("VWA_HIPCC_EXTRA", "").split()  # (utils/env.py Settings documents it; build.py stays import-light)  # (experiments)
    jobs_list = []
    objs = []
    for src in kern_src:
        obj = os.path.join(BUILD, os.path.basename(src) + ".o")
        objs.append(obj)
        if force or not _newer(obj, _deps(src)):
            jobs_list.append(common + ["-c", src, "-o", obj])
    for name in ("bindings", "bindings_stack", "bindings_mixers"):
        src, obj = os.path.join(CSRC, name + ".cpp"), os.path.join(BUILD, name + ".o")
        objs.append(obj)
        if force or not _newer(obj, _deps(src)):
            cmd = common + ["-c", src, "-o", obj, f"-D_GLIBCXX_USE_CXX11_ABI={abi}",
                            "-DTORCH_EXTENSION_NAME=_vwa_kernels", "-DUSE_ROCM=1", "-I", _py_include()]
            for i in inc:
                cmd += ["-I", i]
            jobs_list.append(cmd)
    if core:
        stub_src = os.path.join(CSRC, "core_stubs.cpp")
        stub_obj = os.path.join(BUILD, "core_stubs.o")
        objs.append(stub_obj)
        if force or not _newer(stub_obj, _deps(stub_src)):
            jobs_list.append(common + ["-c", stub_src, "-o", stub_obj])
    with cf.ThreadPoolExecutor(max_workers=jobs) as ex:
        list(ex.map(_run, jobs_list))
    if force or jobs_list or not _newer(target, objs):
        link = [HIPCC, f"--offload-arch={ARCH}", "-shared", "-fPIC", "-o", target + ".tmp"] + objs + [
            "-L", lib, "-ltorch", "-ltorch_cpu", "-ltorch_python", "-lc10", "-lc10_hip", "-ltorch_hip",
            f"-Wl,-rpath,{lib}"]
        _run(link)
        os.replace(target + ".tmp", target)
    return target


def ensure_kernels(core: bool = True) -> None:
    """Build a kernel library if this checkout has none that serves: the core one is enough for models
    without chained or persistent launches (``core``)."""
    if os.path.exists(KERNEL_SO) or (core and os.path.exists(CORE_SO)):
        return
    build_kernels(core=core)


def build_native(force: bool = False) -> str:
    """CPU runtime library (grammar engine + block manager) -- g++ / pybind11."""
    srcs = sorted(glob.glob(os.path.join(CSRC, "runtime", "*.cpp")))
    hdrs = glob.glob(os.path.join(CSRC, "runtime", "*.h"))
    if not srcs:
        return ""
    if not force and _newer(NATIVE_SO, srcs + hdrs):
        return NATIVE_SO
    ext = sysconfig.get_config_var("EXT_SUFFIX")  # noqa: F841 (plain .so name is importable)
    cmd = ["g++", "-O3", "-std=c++17", "-shared", "-fPIC", "-fvisibility=hidden", "-I", _py_include(),
           "-I", _pybind_include(), "-I", os.path.join(CSRC, "runtime"), "-o", NATIVE_SO] + srcs
    _run(cmd)
    return NATIVE_SO


def build_all(force: bool = False) -> list[str]:
    out = []
    n = build_native(force)
    if n:
        out.append(n)
    out.append(build_kernels(force))
    return out


if __name__ == "__main__":
    print(build_all(force="--force" in sys.argv))
