"""In-tree build of the runbooks_amd gfx950 HIP extension.

    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

The built `.so` lands next to the Python package (runbooks_amd/ops/) so it
travels with repo snapshots; there is no JIT cache dependency.
"""
import os
from pathlib import Path

from setuptools import setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from torch.utils import cpp_extension  # noqa: E402

ROOT = Path(__file__).parent
CSRC = ROOT / "runbooks_amd" / "ops" / "csrc"

# One extension module per group, so that a caller can build just what a
# model needs (RB_EXT_GROUPS=core,latent): `core` holds the ops every
# served model runs, `latent` the latent-attention kernels, `shared_kv` the
# attention over rows of keys and values, `lightning` the lightning attention,
# `delta` the delta rules, `streams` the layers around several residual
# streams, `dual` those with norms and input convolutions side by side, `main`
# the rest.
GROUPS = {"core": ("rmsnorm", "layernorm", "glu", "decode_gemm", "sampling"),
          "streams": ("streams", "qkv_prep", "min_gru", "moe"),
          "delta": ("delta", "delta_out", "general_delta"),
          "dual": ("canon", "qkv_conv", "poly_norm")}
PREFIXES = {"shared_kv": "shared_kv", "lightning": "lightning",
            "latent_": "latent"}


def _group_of(stem: str) -> str:
    for group, stems in GROUPS.items():
        if stem in stems:
            return group
    return next((g for p, g in PREFIXES.items() if stem.startswith(p)),
                "main")


MODULES = {"main": ("_hip", "bindings.cpp"),
           **{g: (f"_hip_{g}", f"bindings_{g}.cpp")
              for g in ("core", "latent", "shared_kv", "lightning", "delta",
                        "streams", "dual")}}

# *_hip.hip are build-time copies torch's extension builder leaves behind
kernels = [p for p in sorted(CSRC.glob("*.hip"))
           if not p.stem.endswith("_hip")]
groups = os.environ.get("RB_EXT_GROUPS", ",".join(MODULES)).split(",")

# packed fp32 instructions stay off in device code
HIP_FLAGS = ["-O3", "-std=c++17", "--offload-arch=gfx950",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _extension(group: str):
    module, bindings = MODULES[group]
    return cpp_extension.CUDAExtension(
        name=f"runbooks_amd.ops.{module}",
        sources=[str(p) for p in kernels if _group_of(p.stem) == group]
        + [str(CSRC / bindings)],
        extra_compile_args={"cxx": ["-O3", "-std=c++17"],
                            "nvcc": HIP_FLAGS})


setup(
    name="runbooks_amd",
    version="0.1.0",
    packages=["runbooks_amd"] + [
        f"runbooks_amd.{p}" for p in
        ("api", "cli", "client", "cloud", "controller", "k8s", "models",
         "ops", "parallel", "sci", "serve", "train", "tui", "utils",
         "workloads")],
    entry_points={"console_scripts": [
        # parity: reference cmd/ — sub CLI, controllermanager, sci servers,
        # nbwatch (goreleaser targets .goreleaser.yaml:8-37)
        "sub = runbooks_amd.cli.main:main",
        "runbooks-controller-manager = runbooks_amd.controller.manager:run_manager",
        "sci-kind = runbooks_amd.sci.kind_server:main",
        "sci-gcp = runbooks_amd.sci.gcp_server:main",
        "sci-aws = runbooks_amd.sci.aws_server:main",
        "nbwatch = runbooks_amd.nbwatch:main",
        # kubectl plugin executables (reference kubectl notebook /
        # kubectl applybuild UX — kubectl discovers kubectl-* on PATH)
        "kubectl-notebook = runbooks_amd.cli.main:kubectl_notebook",
        "kubectl-applybuild = runbooks_amd.cli.main:kubectl_applybuild",
    ]},
    ext_modules=[_extension(g) for g in groups],
    cmdclass={"build_ext": cpp_extension.BuildExtension.with_options(use_ninja=True)},
)
