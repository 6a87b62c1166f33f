"""Generalized delta rule: a decay w and a removal rate a per head and key
channel,

    S <- diag(w) S - (a u)(u^T S) + k v^T,   o = S^T r,   u = k / |k|

per head, S [dim, vdim] in fp32; both terms read the old state. Around it:

    y  = [ r heads | k heads | v heads | a logits | gate | bottleneck ]
    y2 = [ decay logits ],   z = [ heads | .. ]

with y2 a product of tanh of y's bottleneck columns, log w = scale
sigmoid(y2 + bias), a = sigmoid(logits + bias).

  * ``tanh_rows``            y's bottleneck columns -> operand of y2
  * ``general_delta_step``   token after token: decoded tokens, short portions
  * ``general_delta_chunk``  long portions in chunks of tokens
  * ``delta_out`` (ops/delta.py): norm per head, weight, sigmoid gate -> z

Sizes per head are padded to a multiple of 8 with zero rows of the packed
weights. A portion that starts at position 0 starts from zero. The chunked
form needs |scale| <= 2: its factors are exponentials of up to a chunk's sum
of log w.

GPU tensors run csrc/general_delta.hip; CPU tensors the plain references
here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .delta import UNIT_EPS
from .latent import _pad_rows, pad_to
from .linear import decode_operand

MAX_DIM = 256                  # padded sizes per head the kernels run


@dataclass(frozen=True)
class GeneralDeltaLayout:
    """Columns of y, y2 and z of one layer (sizes local to this rank)."""
    heads: int
    dim: int
    vdim: int
    rank: int

    @property
    def dc(self):
        return pad_to(self.dim, 8)

    @property
    def vc(self):
        return pad_to(self.vdim, 8)

    @property
    def off_k(self):
        return self.heads * self.dc

    @property
    def off_v(self):
        return 2 * self.heads * self.dc

    @property
    def off_a(self):
        return self.off_v + self.heads * self.vc

    @property
    def off_g(self):
        return self.off_a + self.heads * self.dc

    @property
    def off_r(self):           # bottleneck
        return self.off_g + self.heads * self.vc

    @property
    def n_r(self):
        return pad_to(self.rank, 32)

    @property
    def n_y(self):
        return self.off_r + self.n_r

    @property
    def n_y2(self):
        return pad_to(self.heads * self.dc, 32)

    @property
    def n_o(self):
        return self.heads * self.vc


def pack_in(lay: GeneralDeltaLayout, r, k, v, a, g, w1):
    """Rows of the joint projection, in y's layout."""
    d, e = ((lay.dim,), (lay.dc,)), ((lay.vdim,), (lay.vc,))
    parts = [_pad_rows(w, lay.heads, *s) for w, s in
             ((r, d), (k, d), (v, e), (a, d), (g, e))]
    return torch.cat(parts + [torch.nn.functional.pad(
        w1, (0, 0, 0, lay.n_r - lay.rank))])


def pack_second(lay: GeneralDeltaLayout, w2):
    """[n_y2, n_r]: decay logits from the bottleneck."""
    w = w2.new_zeros(lay.n_y2, lay.n_r)
    w[:lay.off_k, :lay.rank] = _pad_rows(w2, lay.heads, (lay.dim,),
                                         (lay.dc,))
    return w


def pack_bias(lay: GeneralDeltaLayout, w0, a):
    """[2, heads * dc] fp32: biases of the decay and the removal logits."""
    return torch.stack([_pad_rows(b.float()[:, None], lay.heads, (lay.dim,),
                                  (lay.dc,))[:, 0] for b in (w0, a)])


def pack_norm(lay: GeneralDeltaLayout, w):
    """[heads * vc] fp32."""
    return _pad_rows(w.float()[:, None], lay.heads, (lay.vdim,),
                     (lay.vc,))[:, 0].contiguous()


def alloc_general_delta_state(slots: int, lay: GeneralDeltaLayout, device):
    return torch.zeros(slots, lay.heads, lay.dc, lay.vc, device=device)


def tanh_rows(y, off: int, n: int, operand: bool):
    """tanh of n columns of y; operand=True also attaches the decode GEMM's
    operand."""
    if not _backend.use_hip(y):
        return torch.tanh(y[:, off:off + n].float()).to(y.dtype)
    out = torch.empty(y.shape[0], n, dtype=y.dtype, device=y.device)
    swz = decode_operand(y.shape[0], n, y) if operand else None
    _backend.ext().tanh_rows(y, off, out, swz)
    if operand:
        out._rb_swz = swz
    return out


def _recur_ref(y, y2, lay, bias, scale, state, batch, o, seqs):
    H, d, e = lay.heads, lay.dc, lay.vc
    for b in seqs:
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        T, slot = t1 - t0, int(batch.state_slots[b])
        S = state[slot] * float(int(batch.positions[t0]) != 0)

        def part(at, n):
            return y[t0:t1, at:at + H * n].float().view(T, H, n)

        r, k, v = part(0, d), part(lay.off_k, d), part(lay.off_v, e)
        a = torch.sigmoid(part(lay.off_a, d) + bias[1].view(H, d))
        w = torch.exp(scale * torch.sigmoid(
            y2[t0:t1, :H * d].float().view(T, H, d) + bias[0].view(H, d)))
        u = k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + UNIT_EPS)
        for t in range(T):
            seen = torch.einsum("hdv,hd->hv", S, u[t])
            S = w[t][:, :, None] * S - (a[t] * u[t])[:, :, None] * \
                seen[:, None] + k[t][:, :, None] * v[t][:, None]
            o[t0 + t] = torch.einsum("hdv,hd->hv", S, r[t]).reshape(-1)
        state[slot] = S


def general_delta_step(y, y2, lay, bias, scale, state, batch, o):
    """o's rows and the new states of the batch's short portions."""
    if not _backend.use_hip(y):
        return _recur_ref(y, y2, lay, bias, scale, state, batch, o,
                          range(batch.n_short))
    _backend.ext().general_delta_step(
        y, y2, bias, scale, state, batch.positions, batch.cu_q,
        batch.state_slots, o, batch.n_short)


def general_delta_chunk_supported(lay: GeneralDeltaLayout, dtype) -> bool:
    return dtype == torch.bfloat16 and max(lay.dc, lay.vc) <= MAX_DIM


def general_delta_chunk(y, y2, lay, bias, scale, state, batch, o):
    """The same for the long portions."""
    n = batch.n_seqs - batch.n_short
    if not _backend.use_hip(y):
        return _recur_ref(y, y2, lay, bias, scale, state, batch, o,
                          range(batch.n_short, batch.n_seqs))
    _backend.ext().general_delta_chunk(
        y, y2, bias, scale, state, batch.positions, batch.cu_q,
        batch.state_slots, o, batch.n_short, n, batch.max_q_long)
