"""Attention on keys and values of their own, over the paged rows of
ops/shared_kv.py: queries and keys that are normed and rotated, or that pass,
with the values, a short causal convolution.

Around one projection `y` and one output projection that reads `z`:

    y = [ q heads | k heads | v heads | .. ],   z = [ heads of the result | .. ]

  * ``qkv_prep``  RMS norms and rotations of q (in y) and k, cache write
  * ``qkv_conv``  biases and convolutions of q (to a tensor of its own), k
    and v, cache write, the convolutions' last inputs to the slots

then shared_kv_attend and shared_kv_flash. With several maps a head has a
query, and a kv head a key, for each, all with the kv head's value. A cached
row is [ keys | value ]; sizes per head are padded to a multiple of 8 with
zero rows of the packed weight.

GPU tensors run csrc/qkv_prep.hip and csrc/qkv_conv.hip; CPU tensors the plain
references here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .canon import history_ref
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
    rot: int = 0               # rotated dimensions
    maps: int = 1              # attention maps per head

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
        return self.voff + self.vc

    @property
    def voff(self):            # first column of the value in a row
        return self.maps * self.hc

    @property
    def off_k(self):
        return self.heads * self.maps * self.hc

    @property
    def off_v(self):
        return self.off_k + self.kv_heads * self.maps * self.hc

    @property
    def n_y(self):
        return self.off_v + self.kv_heads * self.vc

    @property
    def n_z(self):
        return self.heads * self.vc


def pack_qkv(lay: QKVLayout, q, k, v):
    """Rows of the joint projection, in y's layout."""
    m = lay.maps
    return torch.cat([_pad_rows(q, lay.heads * m, (lay.dim,), (lay.hc,)),
                      _pad_rows(k, lay.kv_heads * m, (lay.dim,), (lay.hc,)),
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


def _conv_ref(y, lay, bias, conv_w, tails, batch, cache, q):
    T, n = y.shape[0], lay.n_y
    out = torch.empty(T, n)
    for b in range(batch.n_seqs):
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        slot, p0 = int(batch.state_slots[b]), int(batch.positions[t0])
        rows = history_ref(y[t0:t1, :n].float(), tails[slot], p0)
        pos = torch.arange(p0 - rows.shape[0] + t1 - t0, p0 + t1 - t0)
        u = rows + bias * (pos >= 0)[:, None]     # none before the start
        out[t0:t1] = sum(u[j:j + t1 - t0] * w for j, w in enumerate(conv_w))
        tails[slot] = rows[t1 - t0:].to(tails.dtype)
    q.copy_(out[:, :lay.off_k])
    s = batch.slots.long()
    cache[s // BLOCK_SIZE, :, s % BLOCK_SIZE] = torch.cat(
        [out[:, lay.off_k:lay.off_v].view(T, lay.kv_heads, lay.voff),
         out[:, lay.off_v:].view(T, lay.kv_heads, lay.vc)],
        dim=-1).to(cache.dtype)


def alloc_conv_tails(slots: int, taps: int, lay: QKVLayout, device, dtype):
    """The last projections of every slot, the oldest first."""
    return torch.zeros(slots, taps - 1, lay.n_y, device=device, dtype=dtype)


def qkv_conv(y, lay: QKVLayout, bias, conv_w, tails, batch, cache):
    """Adds the biases [n_y] to y's first columns and convolves them over
    time with conv_w [taps, n_y] (both fp32). Returns q [T, off_k]; keys and
    values go to `cache`. Afterwards `tails` holds the sequences' last
    projections (without biases)."""
    q = torch.empty(y.shape[0], lay.off_k, dtype=y.dtype, device=y.device)
    if not _backend.use_hip(y):
        _conv_ref(y, lay, bias, conv_w, tails, batch, cache, q)
        return q
    _backend.ext().qkv_conv(
        y, bias, conv_w, tails, batch.positions, batch.cu_q,
        batch.state_slots, batch.seq_of, batch.slots, batch.single,
        batch.n_seqs, cache, lay.voff, q)
    return q
