"""RMS norm of a 32-bit residual and, behind it, a causal convolution over
time that adds to the normed input, for one or more sublayers that read the
same residual:

    n_t = x_t / rms(x_t),   h_t = w n_t + sum_j c_j w n_(t - taps + 1 + j)

w (the norm's weight) and c (the taps) are fixed, so a sublayer is one set of
coefficients, h_t = sum_j f_j n_(t - taps + 1 + j), and all sublayers share n
and the last taps - 1 of them that a sequence's slot keeps, in fp32.

  * single tokens: one kernel does everything
  * portions: the norm's factors, the convolution, then the slots

GPU tensors run csrc/canon.hip; CPU tensors the plain references here.
"""
from __future__ import annotations

import torch

from . import _backend
from .latent import pad_to
from .linear import decode_operand


def pack_coefficients(norms, convs) -> torch.Tensor:
    """[sublayers, taps, D] fp32 from the norms' weights (as they multiply)
    and the convolutions' [D, taps]."""
    out = []
    for w, c in zip(norms, convs):
        f = c.float().t().clone()
        f[-1] += 1
        out.append(f * w.float())
    return torch.stack(out).contiguous()


def alloc_canon_tails(slots: int, taps: int, width: int, device):
    """The last normed inputs of every slot, the oldest first."""
    return torch.zeros(slots, taps - 1, width, device=device)


def history_ref(new, tail, start: int):
    """Inputs of a convolution over a portion that starts at position
    `start`: what came before it (zeros before position 0), then its own
    rows."""
    n = tail.shape[0]
    real = torch.arange(start - n, start) >= 0
    return torch.cat([torch.where(real[:, None], tail.float(), 0.0), new])


def _canon_ref(x, delta, coef, tails, batch, eps, dtype):
    if delta is not None:
        x += delta.float() if delta.dim() == 2 else delta.sum(0)
    n = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    D, taps = x.shape[1], coef.shape[1]
    out = [torch.zeros(x.shape[0], pad_to(D, 32), dtype=dtype)
           for _ in range(coef.shape[0])]
    for b in range(batch.n_seqs):
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        slot = int(batch.state_slots[b])
        rows = history_ref(n[t0:t1], tails[slot], int(batch.positions[t0]))
        for h, f in zip(out, coef):
            h[t0:t1, :D] = sum(rows[j:j + t1 - t0] * f[j]
                               for j in range(taps)).to(dtype)
        tails[slot] = rows[t1 - t0:]
    return out


def canon_norm(x, delta, coef, tails, batch, eps: float, dtype, operands):
    """x [T, D] fp32 += delta in place; the sublayers' inputs in `dtype`,
    [T, D padded to 32] each. delta as in rmsnorm_res32. operands: per
    sublayer, whether to attach the decode GEMM's operand (T <= 32).
    Afterwards `tails` holds the sequences' last normed inputs."""
    if not _backend.use_hip(x):
        return _canon_ref(x, delta, coef, tails, batch, eps, dtype)
    T, D = x.shape
    width = pad_to(D, 32)
    out = [torch.empty(T, width, dtype=dtype, device=x.device)
           for _ in operands]
    swz = [decode_operand(T, width, h) if o else None
           for h, o in zip(out, operands)]
    _backend.ext().canon_norm(
        x, None if delta is None else delta.contiguous(), coef, tails,
        batch.positions, batch.cu_q, batch.state_slots, batch.seq_of,
        batch.single, batch.n_seqs, eps, out, [s for s in swz if s is not None],
        list(operands))
    for h, s in zip(out, swz):
        if s is not None:
            h._rb_swz = s
    return out
