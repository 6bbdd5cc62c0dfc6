"""In-tree hipcc build of the quoracle_amd HIP extensions (gfx950).

Three modules, each one translation unit, built directly with hipcc (no JIT
cache — the .so files must travel with the repo snapshot to the GPU box):

  _quoracle_ops     the Llama-family kernels and their forward driver
  _quoracle_hybrid  recurrent/local-attention mixers and the hybrid driver
  _quoracle_latent  latent attention, mixtures of experts and the same driver

They are separate so that a process serving one family compiles and loads
only that family's kernels.  hipcc cross-compiles gfx950 without a GPU, so
this runs in CPU-only CI too.
"""

from __future__ import annotations

import os
import subprocess
import sys
import sysconfig
import tempfile
from typing import Dict, List, Optional, Sequence

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950")

# module -> (binding source, files it includes)
MODULES: Dict[str, Sequence[str]] = {
    "_quoracle_ops": (
        "bindings.cpp", "common.h", "forward.h", "attention.hip",
        "attention_mfma.hip", "attention_core.h", "elementwise.hip"),
    "_quoracle_hybrid": (
        "hybrid_bindings.cpp", "common.h", "hybrid_common.h", "hybrid_host.h",
        "stream_kernels.hip", "attention_core.h", "attention_local.hip",
        "linear_attention.hip", "hybrid_elementwise.hip", "hybrid_forward.h",
        "hybrid_blocks.h"),
    "_quoracle_latent": (
        "latent_bindings.cpp", "common.h", "hybrid_common.h", "hybrid_host.h",
        "stream_kernels.hip", "latent_elementwise.hip", "grouped_gemm.hip",
        "latent_attention.hip", "moe.hip", "hybrid_forward.h",
        "latent_blocks.h"),
}


def so_path(module: str) -> str:
    return os.path.join(HERE, module + ".so")


SO_PATH = so_path("_quoracle_ops")


def _torch_paths():
    import torch
    from torch.utils import cpp_extension
    includes = cpp_extension.include_paths()
    lib_dir = os.path.join(os.path.dirname(torch.__file__), "lib")
    abi = int(torch._C._GLIBCXX_USE_CXX11_ABI)
    return includes, lib_dir, abi


def _command(module: str, out: str) -> List[str]:
    includes, lib_dir, abi = _torch_paths()
    py_include = sysconfig.get_paths()["include"]
    cmd = [
        "hipcc", "-x", "hip", f"--offload-arch={ARCH}",
        "-O3", "-std=c++17", "-fPIC", "-shared",
        f"-DTORCH_EXTENSION_NAME={module}",
        "-DTORCH_API_INCLUDE_EXTENSION_H",
        "-DUSE_ROCM=1", "-D__HIP_PLATFORM_AMD__=1",
        f"-D_GLIBCXX_USE_CXX11_ABI={abi}",
        "-fno-gpu-rdc",
        # no packed FP32 instructions: some of their forms have given wrong
        # results on this hardware (the host pass warns that it does not
        # know the feature; that is harmless)
        "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
        "-Wno-unused-result",
        "-Wno-inline-asm",      # M0 among the clobbers is meant
    ]
    for inc in includes + [py_include, CSRC]:
        cmd.append(f"-I{inc}")
    cmd.append(os.path.join(CSRC, MODULES[module][0]))
    cmd += [f"-L{lib_dir}", "-ltorch", "-ltorch_cpu", "-ltorch_hip",
            "-lc10", "-lc10_hip", "-ltorch_python", "-lamdhip64",
            f"-Wl,-rpath,{lib_dir}",
            "-o", out]
    return cmd


def _fresh(module: str) -> bool:
    path = so_path(module)
    if not os.path.exists(path):
        return False
    newest = max(os.path.getmtime(os.path.join(CSRC, f))
                 for f in MODULES[module])
    return os.path.getmtime(path) >= newest


def build(force: bool = False, verbose: bool = True,
          modules: Optional[Sequence[str]] = None) -> str:
    """Build the named modules (default: all), side by side; each .so is
    put in place only when it is complete."""
    todo = [m for m in (modules or MODULES) if force or not _fresh(m)]
    jobs = []
    for module in todo:
        fd, part = tempfile.mkstemp(dir=HERE, prefix="." + module,
                                    suffix=".part")
        os.close(fd)
        cmd = _command(module, part)
        if verbose:
            print("[ops.build]", " ".join(cmd), file=sys.stderr, flush=True)
        jobs.append((module, part, cmd, subprocess.Popen(
            cmd, stdout=sys.stderr, stderr=sys.stderr)))
    failed = None
    for module, part, cmd, proc in jobs:
        if proc.wait() == 0:
            os.chmod(part, 0o755)
            os.replace(part, so_path(module))
        else:
            os.unlink(part)
            failed = failed or (proc.returncode, cmd)
    if failed:
        raise subprocess.CalledProcessError(*failed)
    return SO_PATH


if __name__ == "__main__":
    build(force="--force" in sys.argv,
          modules=[a for a in sys.argv[1:] if not a.startswith("-")] or None)
    print(SO_PATH)
