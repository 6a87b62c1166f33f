"""minGRU: a gated recurrence whose gates read only the current token.

    z = sigmoid(y_z + b_z),  u = y_x + b_x,
    c = u + 1/2 where u >= 0, sigmoid(u) elsewhere,
    S <- (1 - z) S + z c,    result = scale S silu(y_g)

on the columns [ z | x | gate ] of a projection y, each `width` padded to a
multiple of 8. The state is fp32, [slots, padded width]; a portion that
starts at position 0 starts from zero.

  * ``min_gru_step``  token after token: decoded tokens, short portions
  * ``min_gru_scan``  long portions, token segments in parallel

GPU tensors run csrc/min_gru.hip; CPU tensors the plain reference here.
"""
from __future__ import annotations

import torch

from . import _backend


def _gru_ref(y, off, bias, state, batch, z, z_off, scale, seqs):
    R = state.shape[1]
    for b in seqs:
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        rows = y[t0:t1].float()
        zt = torch.sigmoid(rows[:, off:off + R] + bias[0])
        u = rows[:, off + R:off + 2 * R] + bias[1]
        cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
        gate = torch.nn.functional.silu(rows[:, off + 2 * R:off + 3 * R])
        slot = int(batch.state_slots[b])
        S = state[slot] * (int(batch.positions[t0]) != 0)
        for t in range(t1 - t0):
            S = S + zt[t] * (cand[t] - S)
            z[t0 + t, z_off:z_off + R] = (scale * S * gate[t]).to(z.dtype)
        state[slot] = S


def min_gru(y, off: int, bias, state, batch, z, z_off: int, scale: float,
            swz=None) -> None:
    """z's columns from z_off on, and the new states, of the whole batch. off:
    y's first column; bias [2, R] fp32."""
    if not _backend.use_hip(y):
        return _gru_ref(y, off, bias, state, batch, z, z_off, scale,
                        range(batch.n_seqs))
    ext, n_long = _backend.ext(), batch.n_seqs - batch.n_short
    if batch.n_short:
        ext.min_gru_step(y, off, bias, state, batch.positions, batch.cu_q,
                         batch.state_slots, 0, batch.n_short, z, z_off, scale,
                         swz)
    if n_long:
        ext.min_gru_scan(y, off, bias, state, batch.positions, batch.cu_q,
                         batch.state_slots, batch.n_short, n_long, z, z_off,
                         scale, batch.max_q_long)
