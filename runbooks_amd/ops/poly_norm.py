"""Polynomial of norms as an activation,

    act(z) = a N(z) + b N(z^2) + c N(z^3) + e,   N(v) = v / rms(v),

with powers taken element by element and N over all columns of a token, in
32-bit. GPU tensors run csrc/poly_norm.hip; CPU tensors the plain reference
here.
"""
from __future__ import annotations

import torch

from . import _backend


def power_sums(u, ff: int):
    """[T, 3] fp32: sums of z^2, z^4, z^6 over the first ff columns."""
    if not _backend.use_hip(u):
        z = u[:, :ff].float()
        return torch.stack([z.pow(p).sum(-1) for p in (2, 4, 6)], dim=1)
    return _backend.ext().power_sums(u, ff)


def poly_norm(u, ff: int, total: int, act, eps: float, z, off: int,
              swz=None, sums=None):
    """z's columns from `off` on: the activation of u's first ff columns,
    zeros behind it. total: columns of a whole token (ff times the ranks);
    act [4] fp32. `sums`: power_sums over all ranks (None: this rank has all
    columns). swz: z's decode operand, filled likewise."""
    if not _backend.use_hip(u):
        v = u[:, :ff].float()
        if sums is None:
            sums = power_sums(u, ff)
        f = act[:3] * torch.rsqrt(sums / total + eps)
        z[:, off:] = 0
        z[:, off:off + ff] = (
            v * (f[:, 0:1] + v * (f[:, 1:2] + v * f[:, 2:3])) + act[3]
        ).to(z.dtype)
        return
    _backend.ext().poly_norm(u, ff, total, act, eps, z, off, swz, sums)
