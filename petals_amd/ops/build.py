"""Build the HIP extensions IN-TREE (the .so files must travel with the source
tree to GPU boxes): `python -m petals_amd.ops.build [name ...]`.

Cross-compiles for gfx950 (no GPU needed at build time). Five libraries:

  core    the kernels of the llama / bloom / falcon / mixtral families
  latent  latent attention, output norms and routed experts (tulezen); it is
          all that a process serving such a model needs
  hybrid  windowed attention with a distance bias and a sink, gated delta rule,
          input norms (lefulorn); likewise
  recurrent  gated linear attention, latent attention with a rotated key part,
          input norms (soselix); likewise
  scores  attention with capped scores, two maps or sigmoid weights, short
          convolutions ahead of it, PolyNorm (zudarax); likewise
"""

from __future__ import annotations

import os
import shutil
import sys

PKG_DIR = os.path.dirname(os.path.abspath(__file__))
SRC_DIR = os.path.join(PKG_DIR, "csrc")

# name -> (.so next to this file, torch extension name, build folder, sources)
EXTENSIONS = {
    "core": (
        "_hip_ops.so", "petals_amd_hip_ops", "_build",
        ["bindings.cpp", "elementwise.hip", "gemv.hip", "attention.hip", "nf4.hip", "int8.hip", "prefill_attn.hip",
         "moe.hip"],
    ),
    "latent": (
        "_hip_latent.so", "petals_amd_hip_latent", os.path.join("_build", "latent"),
        ["latent_bindings.cpp", "latent_attn.hip", "sublayer.hip", "gemv.hip", "moe.hip"],
    ),
    "hybrid": (
        "_hip_hybrid.so", "petals_amd_hip_hybrid", os.path.join("_build", "hybrid"),
        ["hybrid_bindings.cpp", "paged_attn.hip", "delta.hip", "prenorm.hip", "sublayer.hip", "gemv.hip"],
    ),
    "recurrent": (
        "_hip_recurrent.so", "petals_amd_hip_recurrent", os.path.join("_build", "recurrent"),
        ["recurrent_bindings.cpp", "linear_attn.hip", "latent_attn.hip", "rotary_latent.hip", "prenorm.hip",
         "sublayer.hip", "gemv.hip"],
    ),
    "scores": (
        "_hip_scores.so", "petals_amd_hip_scores", os.path.join("_build", "scores"),
        ["scores_bindings.cpp", "paired_attn.hip", "capped_attn.hip", "sigmoid_attn.hip", "prepare_rows.hip", "prenorm.hip",
         "sublayer.hip", "gemv.hip"],
    ),
}


def so_path(name: str = "core") -> str:
    return os.path.join(PKG_DIR, EXTENSIONS[name][0])


def build(verbose: bool = False, name: str = "core") -> str:
    os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")
    os.environ.setdefault("MAX_JOBS", str(min(8, os.cpu_count() or 4)))
    from torch.utils.cpp_extension import load

    _, ext_name, folder, files = EXTENSIONS[name]
    build_dir = os.path.join(PKG_DIR, folder)
    os.makedirs(build_dir, exist_ok=True)
    # torch's hipify writes `<name>_hip.<ext>` next to each source and skips
    # regeneration based on mtimes; copying the tree can scramble those
    # and leave a stale artifact compiling instead of the real source. Purge
    # them so every build regenerates from the true sources.
    import glob

    for stale in glob.glob(os.path.join(SRC_DIR, "*_hip.*")):
        os.unlink(stale)
    # headers are not among the dependencies that torch writes for hipcc
    newest = max(os.path.getmtime(h) for h in glob.glob(os.path.join(SRC_DIR, "*.h")))
    for obj in glob.glob(os.path.join(build_dir, "*.o")):
        if os.path.getmtime(obj) < newest:
            os.unlink(obj)
    load(
        name=ext_name,
        sources=[os.path.join(SRC_DIR, s) for s in files],
        build_directory=build_dir,
        extra_cflags=["-O3", "-std=c++17"],
        # packed FP32 instructions stay off: some of their forms have given
        # wrong results on these machines
        extra_cuda_cflags=["-O3", "-std=c++17", "-ffast-math", "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"],
        verbose=verbose,
        is_python_module=False,
        is_standalone=False,
        keep_intermediates=True,
    )
    # copy the built .so in-tree under a stable name
    built = os.path.join(build_dir, ext_name + ".so")
    if os.path.exists(built):
        shutil.copy2(built, so_path(name))
    return so_path(name)


if __name__ == "__main__":
    for which in [a for a in sys.argv[1:] if not a.startswith("-")] or list(EXTENSIONS):
        print(f"built {build(verbose='-v' in sys.argv, name=which)}", flush=True)
