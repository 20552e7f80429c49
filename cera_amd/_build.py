"""Build the two native libraries of the package in-tree.

* ``cera_amd/lib/libcera_hip.so``  -- HIP kernels + C-ABI (hipcc, gfx950)
* ``cera_amd/lib/libcera_host.so`` -- CPU host layer: quantizers, GGUF, synthetic models (g++)
* ``cera_amd/lib/libcera_hip_llama.so`` + ``cera_amd/lib/cera-hip`` -- the Model-trait layer
  above the C-ABI and its command-line driver (g++)
* ``cera_amd/lib/libcera_hip_layered.so`` + ``cera_amd/lib/cera-trace`` -- the trace runner with
  only the kernels of the models it loads, linked from the same objects
"""
from __future__ import annotations

import hashlib
import os
import shutil
import subprocess
import sys
from pathlib import Path

PKG = Path(__file__).resolve().parent
ROOT = PKG.parent
LIB_DIR = PKG / "lib"
HIP_LIB = LIB_DIR / "libcera_hip.so"
HOST_LIB = LIB_DIR / "libcera_host.so"
LLAMA_LIB = LIB_DIR / "libcera_hip_llama.so"
CLI_BIN = LIB_DIR / "cera-hip"
LAYERED_LIB = LIB_DIR / "libcera_hip_layered.so"
TRACE_BIN = LIB_DIR / "cera-trace"
HSACO = LIB_DIR / "cera_hip_gfx950.hsaco"

HIP_SRCS = sorted((PKG / "csrc").glob("*.hip"))
# what the layered float models need of csrc/
LAYERED_SRCS = [PKG / "csrc" / f"{n}.hip" for n in ("ctx", "model_api", "layered", "layered_seq", "dense", "sigmoid_attn", "softmax_attn",
                                                      "latent", "conv_norm")]
HOST_SRCS = sorted((PKG / "host").glob("*.cpp"))

# -ffp-contract=off: the parity target never fuses a*b+c implicitly; FMAs in
# the kernels are spelled fmaf().  The packed-fp32 feature is switched off
# because some packed forms have produced wrong results on this hardware pool.
HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-shared",
    "-ffp-contract=off", "-fno-fast-math",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    # MFMA results straight into VGPRs: the GEMM epilogue consumes every accumulator element
    # on the VALU, and the AGPR form would cost one v_accvgpr_read per element on top
    "-mllvm", "-amdgpu-mfma-vgpr-form=1",
    "-Wall", "-Wno-unused-function",
]
HOST_FLAGS = ["-O2", "-std=c++17", "-fPIC", "-shared", "-ffp-contract=off", "-fno-fast-math",
              "-pthread", "-Wall", "-Wextra", "-fvisibility=hidden"]


def hipcc_path() -> str:
    for cand in (os.environ.get("HIPCC"), shutil.which("hipcc"), "/opt/rocm/bin/hipcc"):
        if cand and Path(cand).exists():
            return cand
    raise RuntimeError("hipcc not found")


def _run(cmd, verbose: bool, what: str) -> None:
    r = subprocess.run(cmd, capture_output=True, text=True)
    if verbose or r.returncode:
        print(" ".join(cmd), file=sys.stderr)
        print(r.stdout + r.stderr, file=sys.stderr)
    if r.returncode:
        raise RuntimeError(what)


def compile_hip(srcs, verbose: bool = False, jobs: int = 8) -> list[str]:
    """Compile HIP sources to objects in parallel; returns their paths."""
    from concurrent.futures import ThreadPoolExecutor

    LIB_DIR.mkdir(exist_ok=True)
    obj_dir = LIB_DIR / "obj"
    obj_dir.mkdir(exist_ok=True)
    flags = [f for f in HIPCC_FLAGS if f != "-shared"]

    def compile_one(src: Path) -> str:
        obj = obj_dir / (src.stem + ".o")
        _run([hipcc_path(), *flags, f"-I{ROOT / 'include'}", f"-I{PKG / 'csrc'}", "-c", str(src), "-o", str(obj)],
             verbose, f"hipcc failed on {src.name}")
        return str(obj)

    with ThreadPoolExecutor(max_workers=jobs) as ex:
        return list(ex.map(compile_one, srcs))


def link_hip(objs, out: Path, verbose: bool = False) -> Path:
    _run([hipcc_path(), "--offload-arch=gfx950", "-shared", "-fPIC", *objs, "-o", str(out)], verbose, "hipcc link failed")
    return out


def build_hip(verbose: bool = False, jobs: int = 8) -> Path:
    """Compile every csrc/*.hip to an object (in parallel) and link the C-ABI library."""
    return link_hip(compile_hip(sorted((PKG / "csrc").glob("*.hip")), verbose, jobs), HIP_LIB, verbose)


def build_hsaco(verbose: bool = False) -> Path:
    """The standalone gfx950 code object of the lower ABI (include/cera_hip_kernels.h)."""
    LIB_DIR.mkdir(exist_ok=True)
    flags = [f for f in HIPCC_FLAGS if f not in ("-shared", "-fPIC")]
    cmd = [hipcc_path(), "--genco", "--no-gpu-bundle-output", *flags, f"-I{ROOT / 'include'}", f"-I{PKG / 'csrc'}",
           str(PKG / "csrc" / "lower" / "cera_hip_gfx950.hip"), "-o", str(HSACO)]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if verbose or r.returncode:
        print(" ".join(cmd))
        print(r.stdout + r.stderr)
    if r.returncode:
        raise RuntimeError("hipcc --genco failed")
    return HSACO


def build_host(verbose: bool = False) -> Path:
    LIB_DIR.mkdir(exist_ok=True)
    srcs = sorted((PKG / "host").glob("*.cpp"))
    cmd = ["g++", *HOST_FLAGS, f"-I{ROOT / 'include'}", f"-I{PKG / 'host'}", *map(str, srcs),
           "-o", str(HOST_LIB), "-ldl"]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if verbose or r.returncode:
        print(" ".join(cmd))
        print(r.stdout + r.stderr)
    if r.returncode:
        raise RuntimeError("g++ failed building the host library")
    return HOST_LIB


def build_backend(verbose: bool = False) -> Path:
    """HipLlamaModel + its C face (libcera_hip_llama.so) and the cera-hip driver binary.

    Both link against the two libraries above, found at run time next to themselves.
    """
    common = ["g++", "-O2", "-std=c++17", "-fPIC", "-pthread", "-Wall", "-Wextra", "-fvisibility=hidden",
              f"-I{ROOT / 'include'}", f"-I{PKG / 'host'}", f"-I{PKG / 'backend'}"]
    link = [f"-L{LIB_DIR}", "-lcera_hip", "-lcera_host", "-Wl,-rpath,$ORIGIN"]
    b = PKG / "backend"
    # C++ classes are not exported by the host library: compile them in
    host = [str(PKG / "host" / f) for f in ("gguf.cpp", "json.cpp", "safetensors.cpp")]
    models = [str(b / f) for f in ("hip_device_model.cpp", "hip_llama.cpp", "hip_layered.cpp", "nafevik.cpp", "fidinex.cpp", "load_dir.cpp", "load_model.cpp")]
    cmds = [
        [*common, "-shared", *models, str(b / "hip_llama_capi.cpp"), *host, "-o", str(LLAMA_LIB), *link],
        [*common, str(b / "cli.cpp"), str(b / "trace.cpp"), *models, *host, "-o", str(CLI_BIN), *link],
    ]
    for cmd in cmds:
        _run(cmd, verbose, "g++ failed building the backend layer")
    return LLAMA_LIB


def _trace_sources() -> list[Path]:
    """Every file the trace runner is built from (headers of the same directories included)."""
    files = list(LAYERED_SRCS) + sorted((PKG / "csrc").glob("*.h")) + sorted((ROOT / "include").glob("*.h"))
    return files + sorted((PKG / "host").glob("*.[ch]*")) + sorted((PKG / "backend").glob("*.[ch]*")) + [Path(__file__)]


def _trace_stamp() -> str:
    h = hashlib.sha256()
    for f in _trace_sources():
        h.update(f.name.encode() + b"\0" + f.read_bytes())
    return h.hexdigest()


def build_trace(verbose: bool = False, objs=None, jobs: int = 8) -> Path:
    """The trace runner (cera-trace) and the library it runs on.  ``objs``: objects of LAYERED_SRCS
    when they are compiled already."""
    stamp = _trace_stamp()
    if objs is None:
        objs = compile_hip(LAYERED_SRCS, verbose, jobs)
    link_hip(objs, LAYERED_LIB, verbose)
    b, host = PKG / "backend", PKG / "host"
    srcs = [b / "trace_run.cpp", b / "trace.cpp", b / "hip_device_model.cpp", b / "hip_layered.cpp", b / "nafevik.cpp", b / "fidinex.cpp", b / "load_dir.cpp",
            host / "json.cpp", host / "safetensors.cpp"]
    _run(["g++", "-O2", "-std=c++17", "-fPIC", "-pthread", "-Wall", "-Wextra", "-fvisibility=hidden", f"-I{ROOT / 'include'}",
          f"-I{host}", f"-I{b}", *map(str, srcs), "-o", str(TRACE_BIN), f"-L{LIB_DIR}", "-lcera_hip_layered", "-lcera_host",
          "-Wl,-rpath,$ORIGIN"], verbose, "g++ failed building the trace runner")
    (LIB_DIR / "cera-trace.stamp").write_text(stamp)
    return TRACE_BIN


def ensure_trace() -> Path:
    """The trace runner, built first when it is missing or its sources have changed since."""
    import fcntl

    LIB_DIR.mkdir(exist_ok=True)
    with open(LIB_DIR / ".trace.lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        stamp = LIB_DIR / "cera-trace.stamp"
        built = all(p.exists() for p in (TRACE_BIN, LAYERED_LIB, HOST_LIB, stamp))
        if not built or stamp.read_text() != _trace_stamp():
            build_host()
            build_trace()
    return TRACE_BIN


def build_all(verbose: bool = False) -> None:
    build_host(verbose)
    build_hip(verbose)
    build_hsaco(verbose)
    build_backend(verbose)
    build_trace(verbose, [str(LIB_DIR / "obj" / (p.stem + ".o")) for p in LAYERED_SRCS])


if __name__ == "__main__":
    build_all(verbose=True)
