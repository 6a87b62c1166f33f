"""Residual streams with learned mixing, dynamic-tanh norm, squared ReLU.

Instead of one residual x there are s of them, X [T, s, D] in fp32. A
sublayer reads u = sum_s in[s] X_s through a norm; its result y, times a
factor per column and a sigmoid gate of its own input, comes back as

    X_t <- sum_f mix[f, t] X_f + out[t] scale sigmoid(gate + b) y

A `Pending` holds such a result that has not been added yet:
``streams_norm`` adds it, takes the next sublayer's u and norms it, all in
one pass over X.

GPU tensors run csrc/streams.hip; CPU tensors the plain references here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .latent import pad_to

MAX_STREAMS = 16


class DynamicTanh(torch.nn.Module):
    """tanh(alpha x) * weight + bias: a norm without statistics."""

    def __init__(self, dim: int, dtype=None):
        super().__init__()
        self.weight = torch.nn.Parameter(torch.ones(dim, dtype=dtype))
        self.bias = torch.nn.Parameter(torch.zeros(dim, dtype=dtype))
        self.alpha = torch.nn.Parameter(torch.full((), 0.5, dtype=dtype))

    def packed(self) -> torch.Tensor:
        """[2 D + 1] fp32: weight, bias, alpha."""
        return torch.cat([self.weight.data.float(), self.bias.data.float(),
                          self.alpha.data.float().view(1)])


@dataclass
class Pending:
    """A sublayer's result on its way to the streams."""
    delta: torch.Tensor            # fp32 [T, D] or parts [n, T, D]
    extra: torch.Tensor | None     # further parts, likewise
    y: torch.Tensor                # [T, ..]: gate logits from column `off`
    off: int
    join: torch.Tensor             # [2 D + s + s s] fp32: scale, gate bias,
    #                                out, mix

    def rows(self, index) -> "Pending":
        """The same for some of the tokens."""
        def pick(d):
            return None if d is None else d.index_select(d.dim() - 2, index)
        return Pending(pick(self.delta), pick(self.extra),
                       self.y.index_select(0, index), self.off, self.join)


def pack_join(scale, gate_bias, out, mix, mult: float) -> torch.Tensor:
    """Pending.join; the residual factor goes into `out`."""
    return torch.cat([scale.float(), gate_bias.float(), out.float() * mult,
                      mix.float().reshape(-1)])


def _total(delta):
    return delta.float() if delta.dim() == 2 else delta.float().sum(0)


def _streams_norm_ref(x, p, inp, norm, dtype):
    T, s, D = x.shape
    if p is not None:
        scale, bias, out = p.join[:D], p.join[D:2 * D], p.join[2 * D:][:s]
        mix = p.join[2 * D + s:].view(s, s)
        y = _total(p.delta)
        if p.extra is not None:
            y = y + _total(p.extra)
        y = y * scale * torch.sigmoid(p.y[:, p.off:p.off + D].float() + bias)
        x.copy_(torch.einsum("tfd,fg->tgd", x, mix) +
                out[None, :, None] * y[:, None])
    u = torch.einsum("tsd,s->td", x, inp)
    w, b, alpha = norm[:D], norm[D:2 * D], norm[2 * D]
    h = torch.zeros(T, pad_to(D, 32), dtype=dtype)
    h[:, :D] = (torch.tanh(alpha * u) * w + b).to(dtype)
    return h


def streams_norm(x, pending: Pending | None, inp, norm, dtype,
                 operand: bool = False):
    """x [T, s, D] fp32 takes `pending` in place; returns the normed input of
    the next sublayer in `dtype`, [T, D padded to 32] with zero padding. inp
    [s] fp32; norm: DynamicTanh.packed(). operand=True also attaches the
    decode GEMM's operand."""
    if not _backend.use_hip(x):
        return _streams_norm_ref(x, pending, inp, norm, dtype)
    p = pending
    h, swz = _backend.ext().streams_norm(
        x, p and p.delta, p and p.extra, p and p.y, p.off if p else 0,
        p and p.join, inp, norm, dtype == torch.bfloat16, operand)
    if operand:
        h._rb_swz = swz
    return h


def squared_relu(y, n: int, operand: bool = False):
    """relu(y[:, :n])^2 as a matrix of its own (n % 16 == 0)."""
    if not _backend.use_hip(y):
        return (torch.relu(y[:, :n].float()) ** 2).to(y.dtype)
    z, swz = _backend.ext().squared_relu(y, n, operand)
    if operand:
        z._rb_swz = swz
    return z
