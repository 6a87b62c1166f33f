"""Build missing extension modules of a source checkout, in-tree."""
from __future__ import annotations

import fcntl
import os
import subprocess
import sys
from pathlib import Path

_OPS = Path(__file__).parent
_ROOT = _OPS.parent.parent
_MODULE = {"main": "_hip", **{g: f"_hip_{g}" for g in (
    "core", "latent", "shared_kv", "lightning", "delta", "streams", "dual")}}


def _missing(groups) -> list[str]:
    return [g for g in groups
            if not list(_OPS.glob(_MODULE[g] + ".*.so"))]


def ensure_built(groups) -> None:
    """Compile the kernel groups (setup.py) that are not built yet; calls
    in parallel wait for the first one."""
    if not _missing(groups):
        return
    (_ROOT / "build").mkdir(exist_ok=True)
    with open(_ROOT / "build" / ".lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        todo = _missing(groups)
        if todo:
            subprocess.run(
                [sys.executable, "setup.py", "build_ext", "--inplace"],
                cwd=_ROOT, check=True, stdout=sys.stderr,
                env=dict(os.environ, RB_EXT_GROUPS=",".join(todo),
                         PYTORCH_ROCM_ARCH="gfx950"))
