"""Mixture of squared-ReLU experts.

    s = softmax(logits);  chosen = the `top` largest of s + correction, out of
    the `keep` groups of neighbours with the largest entries;
    result = sum over the chosen of s_e down_e(relu(up_e h)^2)

  * ``moe_route``  logits -> chosen experts and their weights
  * ``moe_plan``   (token, choice) pairs sorted by expert, in tiles
  * ``moe_up``     activations of all pairs
  * ``moe_down``   weighted results, one part [tokens, D] per choice (fp32)

The parts are added by whoever takes the result (ops/streams.py). Nothing is
read back by the host, so a step can be captured.

GPU tensors run csrc/moe.hip; CPU tensors the plain references here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend

MAX_EXPERTS = 1024
MAX_TOP = 64


@dataclass
class MoEPlan:
    chosen: torch.Tensor           # [T, top] int32
    weights: torch.Tensor          # [T, top] fp32
    pairs: torch.Tensor | None = None    # token * top + choice, by expert
    # [n, 5] expert, first pair, pairs, the expert's first tile and its tiles;
    # the last row counts the used ones
    tiles: torch.Tensor | None = None
    tile: int = 0                  # most pairs of a tile


def _route_ref(logits, correction, top, groups, keep):
    z = logits if logits.dim() == 2 else logits.sum(0)
    s = torch.softmax(z[:, :correction.numel()].float(), dim=-1)
    choice = s + correction
    if keep < groups:
        best = choice.view(len(s), groups, -1).max(-1).values
        kept = torch.zeros_like(best, dtype=torch.bool).scatter_(
            1, best.topk(keep, dim=-1).indices, True)
        choice = choice.masked_fill(
            ~kept.repeat_interleave(choice.shape[1] // groups, dim=1),
            float("-inf"))
    e = choice.topk(top, dim=-1).indices
    return MoEPlan(e.int(), s.gather(1, e))


def moe_route(logits, correction, top: int, groups: int, keep: int
              ) -> MoEPlan:
    """logits fp32 [T, >= experts], or parts of them [n, T, ..]; correction
    [experts] fp32."""
    if not _backend.use_hip(logits):
        return _route_ref(logits, correction, top, groups, keep)
    e, w = _backend.ext().moe_route(logits, correction, top, groups, keep)
    return MoEPlan(e, w)


def tile_rows(pairs: int, experts: int, bf16: bool) -> int:
    """Pairs per tile: small where the work is reading weights."""
    return 128 if bf16 and pairs >= 32 * experts else 16


def moe_plan(plan: MoEPlan, experts: int, bf16: bool) -> MoEPlan:
    """Sort the pairs by expert."""
    if _backend.use_hip(plan.chosen):
        plan.tile = tile_rows(plan.chosen.numel(), experts, bf16)
        plan.pairs, plan.tiles = _backend.ext().moe_plan(
            plan.chosen, experts, plan.tile)
    return plan


def moe_up(h, w, plan: MoEPlan):
    """relu(h w_e^T)^2 of every pair, by pair number: [pairs, F]. h [T, K],
    w [experts, F, K]."""
    if not _backend.use_hip(h):
        top = plan.chosen.shape[1]
        out = h.new_zeros(plan.chosen.numel(), w.shape[1])
        for i, e in enumerate(plan.chosen.reshape(-1).tolist()):
            out[i] = (torch.relu(w[e].float() @ h[i // top].float()) ** 2
                      ).to(h.dtype)
        return out
    return _backend.ext().moe_gemm(h, w, plan.pairs, plan.tiles, plan.weights,
                                   plan.tile, False)


def moe_down(a, w, plan: MoEPlan):
    """[top, T, D] fp32: a pair's activations through its expert's w
    [experts, D, F], times its weight."""
    if not _backend.use_hip(a):
        T, top = plan.chosen.shape
        out = torch.zeros(top, T, w.shape[1])
        for i, e in enumerate(plan.chosen.reshape(-1).tolist()):
            out[i % top, i // top] = plan.weights[i // top, i % top] * (
                w[e].float() @ a[i].float())
        return out
    return _backend.ext().moe_gemm(a, w, plan.pairs, plan.tiles, plan.weights,
                                   plan.tile, True)
