"""Build the bloombee_amd gfx950 HIP extension in-tree.

Invokes hipcc directly (native HIP source — no hipify pass, no CUDA
compatibility layer). The built .so files land in bloombee_amd/ops/, inside the
tree, so that a copy of the tree carries them (a JIT cache under ~/.cache would
stay behind).

Usage:
    python setup.py build_ext --inplace     # or: python setup.py hip
"""
import os
import subprocess
import sys
import sysconfig
from pathlib import Path

ROOT = Path(__file__).resolve().parent
HIP_DIR = ROOT / "bloombee_amd" / "ops" / "hip"
OPS_DIR = ROOT / "bloombee_amd" / "ops"
# module -> source. _hip_ragged holds what all ragged-batch models need,
# _hip_mixers latent attention and gated linear attention, _hip_recurrent the
# matrix memory and the gated linear recurrent unit, _hip_differential differential
# attention, _hip_hgrn gated linear attention that writes what it forgets.
MODULES = {"_hip_ops": "ext.hip", "_hip_ragged": "ext_ragged.hip",
           "_hip_mixers": "ext_mixers.hip",
           "_hip_recurrent": "ext_recurrent.hip",
           "_hip_differential": "ext_differential.hip",
           "_hip_hgrn": "ext_hgrn.hip"}
ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950")


def torch_paths():
    import torch

    tdir = Path(torch.__file__).parent
    return tdir / "include", tdir / "lib"


def _compile(module: str, source: str, verbose: bool) -> Path:
    """One extension module from one source file."""
    tinc, tlib = torch_paths()
    py_inc = sysconfig.get_paths()["include"]
    out = OPS_DIR / f"{module}.so"
    # private names until the finished file is moved into place: a second
    # process that builds or loads meanwhile never sees a half-written one
    obj = HIP_DIR / f"{source}.{os.getpid()}.o"
    part = OPS_DIR / f".{module}.{os.getpid()}.so"
    compile_cmd = [
        "/opt/rocm/bin/hipcc",
        f"--offload-arch={ARCH}",
        "-O3", "-std=c++17", "-fPIC", "-fno-gpu-rdc",
        # packed FP32 instructions off: some of their forms are unreliable
        "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
        "-I", str(tinc),
        "-I", str(tinc / "torch" / "csrc" / "api" / "include"),
        "-I", "/opt/rocm/include",
        "-I", py_inc,
        "-D__HIP_PLATFORM_AMD__=1", "-DUSE_ROCM=1", "-DHIPBLAS_V2",
        "-DCUDA_HAS_FP16=1", "-D__HIP_NO_HALF_OPERATORS__=1",
        "-D__HIP_NO_HALF_CONVERSIONS__=1", "-DHIP_ENABLE_WARP_SYNC_BUILTINS=1",
        "-DTORCH_API_INCLUDE_EXTENSION_H", f"-DTORCH_EXTENSION_NAME={module}",
        "-c", str(HIP_DIR / source), "-o", str(obj),
    ]
    link_cmd = [
        "g++", "-shared", str(obj),
        "-L", str(tlib), "-L", "/opt/rocm/lib",
        "-lc10", "-ltorch", "-ltorch_cpu", "-ltorch_python",
        "-lamdhip64", "-lc10_hip", "-ltorch_hip", "-lz",
        "-o", str(part),
    ]
    try:
        for cmd in (compile_cmd, link_cmd):
            if verbose:
                print("+", " ".join(cmd), file=sys.stderr)
            subprocess.run(cmd, check=True)
        os.replace(part, out)
    finally:
        obj.unlink(missing_ok=True)
        part.unlink(missing_ok=True)
    return out


def build(modules=None, verbose: bool = True) -> list:
    """Compile the named extension modules (default: all), side by side."""
    from concurrent.futures import ThreadPoolExecutor

    names = list(modules or MODULES)
    with ThreadPoolExecutor(len(names)) as ex:
        return list(ex.map(lambda m: _compile(m, MODULES[m], verbose), names))


if __name__ == "__main__":
    if len(sys.argv) > 1 and sys.argv[1] in ("hip", "build_ext"):
        build()
    else:
        print(__doc__)
