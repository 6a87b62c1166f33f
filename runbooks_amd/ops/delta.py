"""Gated delta rule with one decay per head and key channel.

    S <- g S,  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q

per head, S [dim, vdim] in fp32. q, k, v come from a projection y through a
short causal convolution and silu; q and k are then unit vectors. Around it:

    y  = [ q heads | k heads | v heads | beta | bottleneck | .. ]
    y2 = [ decay logits | gate logits ],   z = [ heads ]

with y2 a product of y's bottleneck columns. log g = -exp(a_log)
softplus(logit + bias).

  * ``delta_step``   token after token: decoded tokens, short portions
  * ``delta_chunk``  long portions in chunks of tokens
  * ``delta_out``    norm per head, weight, sigmoid gate -> z; the
                     convolution's last inputs -> the slots

Sizes per head are padded to a multiple of 8 with zero rows of the packed
weights. A sequence's slot holds S [heads, dim, vdim] and the convolution's
last taps - 1 inputs; a portion that starts at position 0 starts from zero.

GPU tensors run csrc/delta.hip; CPU tensors the plain references here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .latent import _pad_rows, pad_to

UNIT_EPS = 1e-6                # under the root of a unit vector's length
MAX_DIM = 256                  # padded sizes per head the kernels run
MAX_VALUE = 1024


@dataclass(frozen=True)
class DeltaLayout:
    """Columns of y, y2 and z of one layer (sizes local to this rank)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    decay_rank: int
    gate_rank: int

    @property
    def dc(self):
        return pad_to(self.dim, 8)

    @property
    def vc(self):
        return pad_to(self.vdim, 8)

    @property
    def off_k(self):
        return self.kv_heads * self.dc

    @property
    def off_v(self):
        return 2 * self.kv_heads * self.dc

    @property
    def off_b(self):           # = channels of the convolution
        return self.off_v + self.heads * self.vc

    @property
    def off_r(self):           # bottleneck
        return self.off_b + pad_to(self.heads, 8)

    @property
    def n_r(self):
        return pad_to(pad_to(self.decay_rank, 8) + self.gate_rank, 32)

    @property
    def n_y(self):
        return self.off_r + self.n_r

    @property
    def off_g(self):           # gate logits in y2
        return self.heads * self.dc

    @property
    def n_y2(self):
        return pad_to(self.heads * (self.dc + self.vc), 32)

    @property
    def n_o(self):
        return self.heads * self.vc


def pack_in(lay: DeltaLayout, q, k, v, b, a1, g1):
    """Rows of the joint projection, in y's layout."""
    def rows(w, n):
        return torch.nn.functional.pad(w, (0, 0, 0, n - w.shape[0]))
    ra = pad_to(lay.decay_rank, 8)
    return torch.cat([
        _pad_rows(q, lay.kv_heads, (lay.dim,), (lay.dc,)),
        _pad_rows(k, lay.kv_heads, (lay.dim,), (lay.dc,)),
        _pad_rows(v, lay.heads, (lay.vdim,), (lay.vc,)),
        rows(b, lay.off_r - lay.off_b), rows(a1, ra),
        rows(g1, lay.n_r - ra)])


def pack_second(lay: DeltaLayout, a2, g2):
    """[n_y2, n_r]: both second products of the bottleneck as one."""
    ra = pad_to(lay.decay_rank, 8)
    w = a2.new_zeros(lay.n_y2, lay.n_r)
    w[:lay.off_g, :lay.decay_rank] = _pad_rows(a2, lay.heads, (lay.dim,),
                                               (lay.dc,))
    w[lay.off_g:lay.off_g + lay.n_o, ra:ra + lay.gate_rank] = _pad_rows(
        g2, lay.heads, (lay.vdim,), (lay.vc,))
    return w


def pack_conv(lay: DeltaLayout, q, k, v):
    """[taps, channels] fp32, channels in y's order."""
    return torch.cat([
        _pad_rows(q, lay.kv_heads, (lay.dim,), (lay.dc,)),
        _pad_rows(k, lay.kv_heads, (lay.dim,), (lay.dc,)),
        _pad_rows(v, lay.heads, (lay.vdim,), (lay.vc,))]
    ).float().t().contiguous()


def pack_decay(lay: DeltaLayout, a_log, dt_bias):
    """fp32: [heads, dc] biases, then [heads] -exp(a_log)."""
    bias = torch.zeros(lay.heads, lay.dc, device=a_log.device)
    bias[:, :lay.dim] = dt_bias.float().view(lay.heads, lay.dim)
    return torch.cat([bias.view(-1), -torch.exp(a_log.float())])


def alloc_delta_state(slots: int, lay: DeltaLayout, device, dtype):
    """(S, last inputs of the convolution) of every slot."""
    return (torch.zeros(slots, lay.heads, lay.dc, lay.vc, device=device),
            torch.zeros(slots, lay.taps - 1, lay.off_b, device=device,
                        dtype=dtype))


def _recur_ref(y, y2, lay, conv_w, decay, state, batch, o, seqs):
    S_all, tails = state
    G, H, n = lay.kv_heads, lay.heads, lay.off_b
    for b in seqs:
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        T, slot = t1 - t0, int(batch.state_slots[b])
        keep = float(int(batch.positions[t0]) != 0)
        S = S_all[slot] * keep
        raw = torch.cat([tails[slot].float() * keep, y[t0:t1, :n].float()])
        x = sum(raw[j:j + T] * conv_w[j] for j in range(lay.taps))
        x = torch.nn.functional.silu(x)

        def unit(a):
            a = a.reshape(T, G, lay.dc)
            a = a * torch.rsqrt(a.pow(2).sum(-1, keepdim=True) + UNIT_EPS)
            return a.repeat_interleave(H // G, dim=1)

        q = unit(x[:, :lay.off_k]) * lay.dim ** -0.5
        k = unit(x[:, lay.off_k:lay.off_v])
        v = x[:, lay.off_v:].reshape(T, H, lay.vc)
        beta = torch.sigmoid(y[t0:t1, n:n + H].float())
        a = y2[t0:t1, :lay.off_g].float().view(T, H, lay.dc)
        g = torch.exp(decay[H * lay.dc:, None] * torch.nn.functional.softplus(
            a + decay[:H * lay.dc].view(H, lay.dc)))
        for t in range(T):
            S = g[t][:, :, None] * S
            u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S,
                                                        k[t]))
            S = S + k[t][:, :, None] * u[:, None]
            o[t0 + t] = torch.einsum("hdv,hd->hv", S, q[t]).reshape(-1)
        S_all[slot] = S
        tails[slot] = raw[T:].to(tails.dtype)


def delta_step(y, y2, lay, conv_w, decay, state, batch, o):
    """o's rows and the new states of the batch's short portions."""
    if not _backend.use_hip(y):
        return _recur_ref(y, y2, lay, conv_w, decay, state, batch, o,
                          range(batch.n_short))
    _backend.ext().delta_step(
        y, y2, conv_w, decay, *state, batch.positions, batch.cu_q,
        batch.state_slots, o, batch.n_short, lay.kv_heads, lay.dim)


def delta_chunk_supported(lay: DeltaLayout, dtype) -> bool:
    return dtype == torch.bfloat16 and lay.dc <= MAX_DIM


def delta_chunk(y, y2, lay, conv_w, decay, state, batch, o):
    """The same for the long portions."""
    n = batch.n_seqs - batch.n_short
    if not _backend.use_hip(y):
        return _recur_ref(y, y2, lay, conv_w, decay, state, batch, o,
                          range(batch.n_short, batch.n_seqs))
    _backend.ext().delta_chunk(
        y, y2, conv_w, decay, *state, batch.positions, batch.cu_q,
        batch.state_slots, o, batch.n_short, n, batch.max_q_long,
        lay.kv_heads, lay.dim)


def delta_out(o, lay, w, gate, z, eps, swz, y, tails, batch, end=None):
    """z = rmsnorm per head(o) * w * sigmoid(gate's columns from lay.off_g),
    zeros behind it up to column `end` (None: all). w fp32, [vc] for every
    head or [heads * vc]. After it the slots hold the last inputs, y's first
    columns, of the convolution (tails None: there is none)."""
    end = z.shape[1] if end is None else end
    if not _backend.use_hip(o):
        T = o.shape[0]
        r = o.view(T, lay.heads, lay.vc)
        r = r * torch.rsqrt(r.pow(2).sum(-1, keepdim=True) / lay.vdim + eps)
        g = torch.sigmoid(gate[:, lay.off_g:lay.off_g + lay.n_o].float())
        z[:, :lay.n_o] = ((r * w.view(-1, lay.vc)).view(T, -1) * g).to(z.dtype)
        z[:, lay.n_o:end] = 0
        return
    _backend.ext().delta_out(o, w, gate, lay.off_g, z, swz, lay.heads,
                             lay.vdim, eps, y, tails, batch.positions,
                             batch.cu_q, batch.state_slots, batch.n_seqs, end)
