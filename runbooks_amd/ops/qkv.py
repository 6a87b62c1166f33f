"""Attention on keys and values of their own, over the paged rows of
ops/shared_kv.py: normed, rotated queries and keys.

Around one projection `y` and one output projection that reads `z`:

    y = [ q heads | k heads | v heads | .. ],   z = [ heads of the result | .. ]

  * ``qkv_prep``  RMS norms and rotations of q (in y) and k, cache write

then shared_kv_attend and shared_kv_flash. A cached row is [ key | value ];
sizes per head are padded to a multiple of 8 with zero rows of the packed
weight.

GPU tensors run csrc/qkv_prep.hip; CPU tensors the plain reference here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .kvcache import BLOCK_SIZE
from .latent import _pad_rows, pad_to, rope_interleaved_ref


@dataclass(frozen=True)
class QKVLayout:
    """Columns of y, z and the cached rows of one layer (sizes local to this
    rank)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    rot: int                   # rotated dimensions

    @property
    def group(self):
        return self.heads // self.kv_heads

    @property
    def hc(self):              # one head of q or k
        return pad_to(self.dim, 8)

    @property
    def vc(self):
        return pad_to(self.vdim, 8)

    @property
    def ec(self):              # one cached row
        return self.hc + self.vc

    @property
    def voff(self):            # first column of the value in a row
        return self.hc

    @property
    def off_k(self):
        return self.heads * self.hc

    @property
    def off_v(self):
        return self.off_k + self.kv_heads * self.hc

    @property
    def n_y(self):
        return self.off_v + self.kv_heads * self.vc

    @property
    def n_z(self):
        return self.heads * self.vc


def pack_qkv(lay: QKVLayout, q, k, v):
    """Rows of the joint projection, in y's layout."""
    return torch.cat([_pad_rows(q, lay.heads, (lay.dim,), (lay.hc,)),
                      _pad_rows(k, lay.kv_heads, (lay.dim,), (lay.hc,)),
                      _pad_rows(v, lay.kv_heads, (lay.vdim,), (lay.vc,))])


def pack_columns(w, groups: int, size: int, padded: int):
    """[N, groups * size] -> [N, groups * padded] with zero columns."""
    out = w.new_zeros(w.shape[0], groups, padded)
    out[:, :, :size] = w.view(w.shape[0], groups, size)
    return out.view(w.shape[0], -1)


def _prep_ref(y, lay, cos, sin, positions, slots, cache, norms, eps):
    T = y.shape[0]

    def head(a, n, w):
        x = y[:, a:a + n * lay.hc].float().view(T, n, lay.hc)[..., :lay.dim]
        x = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w
        out = torch.zeros(T, n, lay.hc)
        out[..., :lay.dim] = x
        out[..., :lay.rot] = rope_interleaved_ref(
            x[..., :lay.rot], cos, sin, positions)
        return out

    q = head(0, lay.heads, norms[0])
    k = head(lay.off_k, lay.kv_heads, norms[1])
    v = y[:, lay.off_v:lay.n_y].float().reshape(T, lay.kv_heads, lay.vc)
    s = slots.long()
    cache[s // BLOCK_SIZE, :, s % BLOCK_SIZE] = torch.cat(
        [k, v], dim=-1).to(cache.dtype)
    y[:, :lay.off_k] = q.reshape(T, -1).to(y.dtype)


def qkv_prep(y, lay: QKVLayout, cos, sin, positions, slots, cache, norms,
             eps: float):
    """Norm and rotate q inside y, write the rows of keys and values to
    `cache` at `slots`. norms [2, dim] fp32: weights of q's and k's norm;
    cos, sin [positions, rot / 2]."""
    if not _backend.use_hip(y):
        return _prep_ref(y, lay, cos, sin, positions, slots, cache, norms,
                         eps)
    _backend.ext().qkv_prep(y, cos, sin, positions, slots, cache, norms,
                            lay.heads, lay.dim, lay.hc, eps)
