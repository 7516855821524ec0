"""Build the HIP libraries (gfx950) in-tree with hipcc.

    python -m omniserve_amd.build [--force]

hipcc cross-compiles without a GPU.  The libraries land next to this file so that they travel with the source tree; objects
go to git-ignored build/ folders beside the sources.

    libomniserve_hip.so        the quantized hot path (csrc/*.hip) behind include/omniserve_hip.h
    libomniserve_lm_bf16.so    the layers of the serving engine's models (csrc/lm/*.hip) behind include/omniserve_lm.h,
    libomniserve_lm_f32.so     the same sources compiled for one element type each, so that a process builds and loads only
                               the one its model runs in
"""
from __future__ import annotations

import contextlib
import os
import shutil
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
INCLUDE = os.path.join(os.path.dirname(HERE), "include")
CSRC = os.path.join(HERE, "csrc")
OBJ = os.path.join(CSRC, "build")
LIB = os.path.join(HERE, "libomniserve_hip.so")
ARCH = "gfx950"
SOURCES = ["qgemm_plan.hip", "qgemm_chn.hip", "qgemm_grp.hip", "qgemm_w8.hip",
           "elementwise.hip", "offpath.hip", "kv_cache.hip", "attn_prefill.hip", "sparse_utils.hip", "tp_comm.hip", "row_dtypes.hip", "norm_gemv_fused.hip"]
# no packed-f32 instructions: some of their forms have returned wrong results on this hardware
NO_PACKED_F32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
# -ffp-contract=off: the fp32 epilogues / quantisers must round exactly like oracle/ (explicit
# fma where wanted).  No -ffast-math anywhere.
FLAGS = ["--offload-arch=" + ARCH, "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off", *NO_PACKED_F32,
         "-Wall", "-Wno-unused-function",
         # qgemm_midm.h's LDS-DMA statements name M0 as clobbered ("reserved register" warning, 1 240 of them per build): the M0
         # discipline of those kernels is asserted on the disassembly instead (tests/test_code_objects_cpu.py)
         "-Wno-inline-asm", "-I" + CSRC, "-I" + INCLUDE]

LM_CSRC = os.path.join(CSRC, "lm")
LM_SOURCES = ["lm_rows.hip", "lm_gemm.hip", "lm_route.hip", "lm_attn.hip", "lm_attn_decode.hip", "lm_linear_attn.hip",
              "lm_latent.hip", "lm_gla.hip", "lm_delta.hip"]
LM_FLAGS = ["--offload-arch=" + ARCH, "-O3", "-std=c++17", "-fPIC", *NO_PACKED_F32, "-Wall", "-Wno-unused-function",
            "-I" + LM_CSRC, "-I" + INCLUDE]
LM_ELEM = {"bf16": 0, "f32": 1}        # -DLM_ELEM=<n>


def _hipcc() -> str:
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(exe):
        raise RuntimeError("hipcc not found: the HIP library cannot be built")
    return exe


def _deps_mtime(*roots) -> float:
    m = 0.0
    for root in roots or (CSRC, INCLUDE):
        for f in os.listdir(root):
            if f.endswith((".hip", ".h", ".cpp")):
                m = max(m, os.path.getmtime(os.path.join(root, f)))
    return max(m, os.path.getmtime(os.path.abspath(__file__)))


EXT_SRC = os.path.join(HERE, "csrc_ext", "omni_ext.cpp")


def ext_path() -> str:
    import sysconfig
    return os.path.join(HERE, "_omni_ext" + sysconfig.get_config_var("EXT_SUFFIX"))


def needs_build() -> bool:
    if not os.path.exists(LIB) or os.path.getmtime(LIB) < _deps_mtime():
        return True
    ext = ext_path()
    return not os.path.exists(ext) or os.path.getmtime(ext) < max(os.path.getmtime(EXT_SRC), os.path.getmtime(LIB))


def build_ext(verbose: bool = False) -> str:
    """The pybind11 fast path of the mirror (csrc_ext/omni_ext.cpp): host-only C++ against the installed torch's headers,
    linked to libomniserve_hip.so next to it (rpath $ORIGIN); g++, ~25 s.  The mirror works without it (ctypes)."""
    import sysconfig
    import torch
    from torch.utils import cpp_extension as ce
    out = ext_path()
    inc = list(ce.include_paths()) + ["/opt/rocm/include", INCLUDE, sysconfig.get_paths()["include"]]
    torch_lib = os.path.join(os.path.dirname(torch.__file__), "lib")
    cmd = [shutil.which("g++") or "g++", "-O2", "-std=c++17", "-fPIC", "-shared", "-D__HIP_PLATFORM_AMD__=1", "-DUSE_ROCM=1",
           "-DTORCH_EXTENSION_NAME=_omni_ext", "-DTORCH_API_INCLUDE_EXTENSION_H",
           "-D_GLIBCXX_USE_CXX11_ABI=%d" % int(torch._C._GLIBCXX_USE_CXX11_ABI)]
    cmd += ["-I" + i for i in inc]
    tmp = out + ".tmp"
    cmd += [EXT_SRC, "-o", tmp, "-L" + torch_lib, "-ltorch", "-ltorch_cpu", "-ltorch_python", "-lc10", "-lc10_hip", "-ltorch_hip",
            "-L" + HERE, "-l:libomniserve_hip.so", "-Wl,-rpath,$ORIGIN", "-Wl,-rpath," + torch_lib]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError("building the pybind11 fast path failed:\n%s" % r.stderr[-4000:])
    os.replace(tmp, out)
    return out


def _compile_and_link(csrc: str, sources, flags, obj_dir: str, lib: str, verbose: bool) -> None:
    os.makedirs(obj_dir, exist_ok=True)
    hipcc = _hipcc()

    def compile_one(src: str) -> str:
        obj = os.path.join(obj_dir, os.path.splitext(src)[0] + ".o")
        extra = os.environ.get("OMNI_HIPCC_EXTRA", "").split()   # tuning experiments only (e.g. -DOMNI_GEMM_MIN_BLOCKS=2)
        cmd = [hipcc, *flags, *extra, "-c", os.path.join(csrc, src), "-o", obj]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError("hipcc failed for %s:\n%s\n%s" % (src, r.stdout, r.stderr))
        err = "\n".join(l for l in r.stderr.splitlines() if "packed-fp32-ops" not in l)     # (the host pass does not know the feature)
        if verbose and err.strip():
            print(err, file=sys.stderr)
        return obj

    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        objs = list(ex.map(compile_one, sources))
    tmp = lib + ".tmp"
    cmd = [hipcc, "--offload-arch=" + ARCH, "-shared", "-fPIC", *objs, "-o", tmp]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError("link failed:\n%s\n%s" % (r.stdout, r.stderr))
    os.replace(tmp, lib)


def build(force: bool = False, verbose: bool = False) -> str:
    if not force and not needs_build():
        return LIB
    if force or not os.path.exists(LIB) or os.path.getmtime(LIB) < _deps_mtime():      # (else: only the binding is stale)
        _compile_and_link(CSRC, SOURCES, FLAGS, OBJ, LIB, verbose)
    try:
        build_ext(verbose)
    except Exception as exc:   # noqa: BLE001  (the mirror works without it: ctypes)
        print("omniserve_amd.build: the pybind11 fast path was not built (%s); the ctypes mirror stays in use" % str(exc)[-400:],
              file=sys.stderr)
    return LIB


def lm_lib_path(elem: str) -> str:
    return os.path.join(HERE, "libomniserve_lm_%s.so" % elem)


@contextlib.contextmanager
def _build_lock():
    """One builder at a time per checkout (two processes may start in a fresh one)."""
    import fcntl
    with open(os.path.join(HERE, ".build.lock"), "w") as f:
        fcntl.flock(f, fcntl.LOCK_EX)
        try:
            yield
        finally:
            fcntl.flock(f, fcntl.LOCK_UN)


def build_lm(elem: str, force: bool = False, verbose: bool = False) -> str:
    """The engine's layer library for one element type ("bf16" or "f32")."""
    lib = lm_lib_path(elem)
    with _build_lock():
        if force or not os.path.exists(lib) or os.path.getmtime(lib) < _deps_mtime(LM_CSRC, INCLUDE):
            _compile_and_link(LM_CSRC, LM_SOURCES, LM_FLAGS + ["-DLM_ELEM=%d" % LM_ELEM[elem]],
                              os.path.join(LM_CSRC, "build", elem), lib, verbose)
    return lib


def build_all(force: bool = False, verbose: bool = False) -> list:
    return [build(force, verbose)] + [build_lm(e, force, verbose) for e in LM_ELEM]


if __name__ == "__main__":
    print("\n".join(build_all(force="--force" in sys.argv, verbose=True)))
