"""Build libfleet_mk.so (HIP kernels + C-ABI host library) for gfx950 with hipcc.

Usage: python build.py            (from anywhere; output lands next to this file: the library, then the Cython binding
                                   mirage/_cython/core.*.so that links against it)

The kernels are translation units of their own (build.KERNELS) and compile side by side.  `build(kernels=...)` makes a
library with only some of them (a graph that needs a missing one is refused by mk_compile); `ensure_library()` is what a
program calls that wants to run one kind of graph from a fresh checkout.
"""
import os
import shutil
import subprocess
import sys
import tempfile
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB = os.path.join(HERE, "libfleet_mk.so")

# kernels of mk_kernel.hip (-DMK_KERNEL_<name>): the fixed-shape pair, the flex ones, those with the mix stages beside them,
# those with the hybrid stages beside both, and those with the dual stages beside flex, norms, routing and experts
KERNELS = ("DENSE", "FLEX", "FLEX_M1", "FLEX_F32", "MIX", "MIX_M1", "MIX_F32", "HYB", "HYB_M1", "HYB_F32", "DUAL", "DUAL_M1", "DUAL_F32")

HIPCC_FLAGS = [
    "--offload-arch=gfx950",
    "-O3",
    "-std=c++17",
    "-fPIC",
    # packed fp32 VALU forms are disabled for all device code
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-Wno-unused-command-line-argument", "-Wno-pass-failed",
]


def _run(cmd, verbose):
    if verbose:
        print(" ".join(cmd), flush=True)
    res = subprocess.run(cmd, cwd=CSRC, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    out = "\n".join(l for l in res.stdout.splitlines() if "packed-fp32-ops" not in l)
    if res.returncode != 0:
        raise RuntimeError("hipcc failed:\n" + out)
    if verbose and out.strip():
        print(out)


def build(verbose: bool = True, defines=(), out: str = None, kernels=KERNELS) -> str:
    hipcc = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(hipcc):
        raise RuntimeError("hipcc not found: the megakernel library cannot be built")
    lib = out or LIB
    extra = ["-D" + d for d in defines]
    with tempfile.TemporaryDirectory(prefix="fleet_mk_build_") as tmp:
        units = [(k.lower(), ["-DMK_KERNEL_" + k, "mk_kernel.hip"]) for k in kernels]
        units.append(("pack", ["mk_pack.hip"]))
        units.append(("host", ["-DMK_HAVE_KERNEL_" + k for k in kernels] + ["-x", "hip", "mk_host.cpp"]))
        objs = [os.path.join(tmp, name + ".o") for name, _ in units]
        workers = min(len(units), int(os.environ.get("MAX_JOBS", "8")))
        with ThreadPoolExecutor(workers) as pool:
            list(pool.map(lambda u: _run([hipcc] + HIPCC_FLAGS + extra + ["-c"] + u[0][1] + ["-o", u[1]], verbose), zip(units, objs)))
        part = os.path.join(os.path.dirname(lib), f".{os.path.basename(lib)}.{os.getpid()}")
        _run([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC"] + objs + ["-o", part], verbose)
        os.replace(part, lib)  # a program that finds the library finds all of it
    return lib


def ensure_library(kernels) -> str:
    """Path of a built library that holds `kernels`: the full one when it is there, else one with exactly these, compiled
    on first use."""
    if os.path.exists(LIB):
        return LIB
    lib = os.path.join(HERE, "libfleet_mk_" + "_".join(k.lower() for k in kernels) + ".so")
    if not os.path.exists(lib):
        print("compiling " + ", ".join(kernels), file=sys.stderr, flush=True)
        build(verbose=False, out=lib, kernels=kernels)
    return lib


def build_cython(verbose: bool = True) -> str:
    """Compile the Cython binding (mirage/_cython/core.pyx -> core.<abi>.so) against include/fleet_mk.h and link it to the
    library next to this file.  Needs the library to be built first."""
    import sysconfig
    cy_dir = os.path.join(HERE, "mirage", "_cython")
    c_file = os.path.join(cy_dir, "core.c")
    out = os.path.join(cy_dir, "core" + sysconfig.get_config_var("EXT_SUFFIX"))
    steps = [
        [sys.executable, "-m", "cython", "-3", "--module-name", "mirage._cython.core", "core.pyx", "-o", c_file],
        [shutil.which("gcc") or "gcc", "-O2", "-fPIC", "-shared", "-Wno-unused-function", "-I" + sysconfig.get_paths()["include"],
         "-I" + os.path.join(os.path.dirname(HERE), "include"), c_file, "-o", out, "-L" + HERE, "-lfleet_mk", "-Wl,-rpath,$ORIGIN/../.."],
    ]
    for cmd in steps:
        if verbose:
            print(" ".join(cmd), flush=True)
        res = subprocess.run(cmd, cwd=cy_dir, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
        if res.returncode != 0:
            raise RuntimeError("building the Cython binding failed:\n" + res.stdout)
    return out


if __name__ == "__main__":
    build()
    print("built", LIB)
    print("built", build_cython())
    sys.exit(0)
