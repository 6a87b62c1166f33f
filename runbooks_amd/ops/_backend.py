"""Backend loader for the gfx950 HIP extension.

Policy (per the framework's no-silent-fallback rule): on a GPU box the
hand-written HIP kernels are THE compute path — if a tensor is on the GPU
and the extension is missing, ops raise instead of silently falling back
to eager PyTorch. On CPU (CI containers have no GPU) ops use plain
PyTorch fp32 reference implementations, which are also what kernel
numerics tests compare against.
"""
from __future__ import annotations

import importlib

import torch

# The kernels are built as several modules (setup.py): ops shared by every
# served model, one per kind of mixer or layer, and the rest.
_MODULES = ("_hip_core", "_hip_latent", "_hip_shared_kv", "_hip_lightning",
            "_hip_delta", "_hip_streams", "_hip_dual", "_hip")
_BUILD_HINT = ("Run `PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext "
               "--inplace` at the repo root.")


class _Extension:
    """All built kernel modules as one namespace. A function whose module
    is not built raises on use, naming the cause."""

    def __init__(self):
        self.mods, self.errors = {}, {}
        for name in _MODULES:
            try:
                self.mods[name] = importlib.import_module(
                    f"runbooks_amd.ops.{name}")
            except Exception as e:  # noqa: BLE001
                self.errors[name] = e

    def __getattr__(self, fn):
        for mod in self.__dict__["mods"].values():
            f = getattr(mod, fn, None)
            if f is not None:
                self.__dict__[fn] = f
                return f
        raise RuntimeError(
            f"runbooks_amd: kernel {fn!r} is in no built gfx950 extension "
            f"module. {_BUILD_HINT} Import errors: {self.errors!r}")


_EXT: _Extension | None = None


def _load():
    global _EXT
    if _EXT is None:
        _EXT = _Extension()
    return _EXT if _EXT.mods else None


def has_hip() -> bool:
    """True when the gfx950 extension is importable AND a GPU is visible."""
    return torch.cuda.is_available() and _load() is not None


def ext():
    """Return the extension namespace; raise loudly if nothing is built."""
    m = _load()
    if m is None:
        raise RuntimeError(
            "runbooks_amd: GPU tensor seen but the gfx950 HIP extension is "
            f"not built. {_BUILD_HINT} Import errors: {_EXT.errors!r}")
    return m


def use_hip(*tensors: torch.Tensor) -> bool:
    """Dispatch decision for an op: any GPU tensor -> HIP path (or raise)."""
    on_gpu = any(t.is_cuda for t in tensors if isinstance(t, torch.Tensor))
    if on_gpu:
        ext()  # raises if missing
        return True
    return False
