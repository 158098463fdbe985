"""In-tree build of the CDNA4 HIP extension (gfx950 only, no hipify).

Drives hipcc directly — no CUDA compatibility layer, no JIT cache: the
resulting ``_C.so`` lives next to this file so the gpurun snapshot carries it.

Three extensions, so that a model family compiles only what it runs:

  core    -> _C.so         transformer kernels
  seqmix  -> _C_seqmix.so  sequence-mixer kernels (ops/seqmix.py)
  moe     -> _C_moe.so     expert-routing kernels (ops.moe_*)

Usage:  python -m fusioninfer_amd.ops.build [core|seqmix|moe|all] [--force]
"""

from __future__ import annotations

import os
import subprocess
import sys
import sysconfig
from concurrent.futures import ThreadPoolExecutor

OPS_DIR = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(OPS_DIR, "csrc")
SO_PATH = os.path.join(OPS_DIR, "_C.so")

SOURCES = [
    "ops.hip",
    "norm.hip",
    "activation.hip",
    "quant.hip",
    "rope.hip",
    "cache.hip",
    "paged_attention.hip",
    "prefill_attention.hip",
]

MOE_SOURCES = [
    "moe_bindings.hip",
    "moe_gemm.hip",
    "moe_plain.hip",
]


SEQMIX_SOURCES = [
    "seqmix_bindings.hip",
    "seqmix_norm.hip",
    "seqmix_attention.hip",
    "seqmix_delta.hip",
    "seqmix_stream.hip",
    "seqmix_linear.hip",
    "seqmix_window.hip",
    "seqmix_parallel.hip",
    "seqmix_sink.hip",
    "seqmix_postnorm.hip",
    "seqmix_hyper.hip",
    "seqmix_memory.hip",
    "seqmix_hyper_bindings.hip",
    "seqmix_sandwich.hip",
    "seqmix_scan.hip",
    "seqmix_scan_bindings.hip",
]

EXTENSIONS = {
    "core": ("_C", SOURCES, ["common.h"]),
    "seqmix": ("_C_seqmix", SEQMIX_SOURCES, ["common.h", "seqmix.h", "seqmix_bind.h",
                "seqmix_hyper.h", "seqmix_scan.h"]),
    "moe": ("_C_moe", MOE_SOURCES, ["common.h", "seqmix.h"]),
}


def extension_path(ext: str) -> str:
    return os.path.join(OPS_DIR, EXTENSIONS[ext][0] + ".so")


def build(verbose: bool = True, force: bool = False) -> str:
    """The core extension (kept as the historical entry point)."""
    return build_extension("core", verbose=verbose, force=force)


def build_extension(ext: str, verbose: bool = True,
                    force: bool = False) -> str:
    import torch
    from torch.utils import cpp_extension as ce

    mod_name, sources, headers = EXTENSIONS[ext]
    so_path = extension_path(ext)
    srcs = [os.path.join(CSRC, s) for s in sources]
    hdrs = [os.path.join(CSRC, h) for h in headers]
    if not force and os.path.exists(so_path):
        so_mtime = os.path.getmtime(so_path)
        if all(os.path.getmtime(f) < so_mtime for f in srcs + hdrs):
            return so_path
    hipcc = os.path.join(os.environ.get("ROCM_PATH", "/opt/rocm"), "bin", "hipcc")
    torch_lib = ce.library_paths()[0]
    common = [
        hipcc,
        "--offload-arch=gfx950",
        "-O3",
        "-std=c++17",
        "-fPIC",
        f"-DTORCH_EXTENSION_NAME={mod_name}",
        # packed-fp32 VALU forms are kept out of generated code
        "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
        "-DTORCH_API_INCLUDE_EXTENSION_H",
        f"-D_GLIBCXX_USE_CXX11_ABI={int(torch._C._GLIBCXX_USE_CXX11_ABI)}",
        *getattr(ce, "COMMON_HIP_FLAGS", ["-D__HIP_PLATFORM_AMD__=1", "-DUSE_ROCM=1"]),
        "-DHIP_ENABLE_WARP_SYNC_BUILTINS",
        *[f"-I{p}" for p in ce.include_paths()],
        f"-I{sysconfig.get_paths()['include']}",
        f"-I{CSRC}",
    ]
    out = None if verbose else subprocess.DEVNULL

    def run(cmd):
        if verbose:
            print("[fusioninfer build]", " ".join(cmd), file=sys.stderr)
        subprocess.run(cmd, check=True, stdout=out, stderr=out)

    # one object per source, compiled side by side; objects newer than their
    # source and all headers are kept unless ``force``
    obj_dir = os.path.join(OPS_DIR, "build", ext)
    os.makedirs(obj_dir, exist_ok=True)
    newest_hdr = max(os.path.getmtime(f) for f in hdrs)

    def compile_one(src):
        obj = os.path.join(obj_dir, os.path.basename(src) + ".o")
        if not force and os.path.exists(obj) and os.path.getmtime(obj) > max(
                os.path.getmtime(src), newest_hdr):
            return obj
        tmp = obj + ".%d.tmp" % os.getpid()
        run(common + ["-c", src, "-o", tmp])
        os.replace(tmp, obj)
        return obj

    jobs = int(os.environ.get("MAX_JOBS") or min(os.cpu_count() or 1, 8))
    with ThreadPoolExecutor(max_workers=max(1, min(jobs, 16))) as pool:
        objs = list(pool.map(compile_one, srcs))
    # link next to the target and rename: a concurrent reader never sees a
    # half-written library
    tmp = so_path + ".%d.tmp" % os.getpid()
    run([
        hipcc,
        "--offload-arch=gfx950",
        "-shared",
        "-fPIC",
        *objs,
        f"-L{torch_lib}",
        f"-Wl,-rpath,{torch_lib}",
        "-ltorch",
        "-ltorch_python",
        "-lc10",
        "-ltorch_hip",
        "-lc10_hip",
        "-lamdhip64",
        "-o",
        tmp,
    ])
    os.replace(tmp, so_path)
    return so_path


if __name__ == "__main__":
    which = [a for a in sys.argv[1:] if not a.startswith("-")] or ["all"]
    names = list(EXTENSIONS) if "all" in which else which
    for name in names:
        print(build_extension(name, force="--force" in sys.argv))
