"""One engine step as a ragged batch: portions of several sequences.

A `StepPlan` is the host-side description (which tokens of which
sequence, its cache blocks, which logits are wanted). It flattens to one
integer vector, so tensor-parallel workers can rebuild it, and turns into
a `RaggedBatch` of device tensors that the model consumes.

Sequences are ordered so that the short portions come first: those run
attention on the cached latents themselves (one pass over the pages per
head group), the longer ones on keys and values expanded from them; other
mixers have a kernel for short portions and one for long ones, too.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np
import torch

# portions of at most this many tokens count as short
ABSORB_MAX = 32


@dataclass
class Portion:
    tokens: list[int]          # the sequence's next tokens
    start: int                 # absolute position of the first of them
    dropped: int               # leading tokens whose blocks were given back
    blocks: list[int]          # blocks of positions dropped, dropped+bs, ...
    want: list[int]            # places among `tokens` whose logits to return
    slot: int = 0              # the sequence's state slot


@dataclass
class RaggedBatch:
    tokens: torch.Tensor       # [T] int64
    positions: torch.Tensor    # [T] int32, absolute (rotation)
    slots: torch.Tensor        # [T] int32, cache slot of each token
    cu_q: torch.Tensor         # [B + 1] int32, first token of each sequence
    seq_lens: torch.Tensor     # [B] int32, retained tokens incl. new ones
    block_tables: torch.Tensor  # [B, n] int32
    state_slots: torch.Tensor  # [B] int32
    seq_of: torch.Tensor       # [T] int32, sequence of each token
    rows: torch.Tensor | None  # token rows whose logits are wanted (None: all)
    n_seqs: int
    # sequences [0, n_short) are short portions
    n_short: int
    t_short: int               # their tokens
    max_q: int                 # their longest portion
    max_keys: int | None       # their longest context (None: unknown)
    # the others, per window: (context slots [Tk], meta [n, 5]); a meta row
    # is (first query row, queries, first key row, keys, key index of the
    # first query)
    long_plans: dict = field(default_factory=dict)
    max_q_long: int = 0

    @property
    def single(self) -> bool:
        """Every portion is one token."""
        return self.n_short == self.n_seqs and self.max_q <= 1


class StepPlan:
    def __init__(self, portions: list[Portion]):
        self.portions = portions

    # -- one integer vector (tensor-parallel broadcast) ---------------------
    def flatten(self) -> torch.Tensor:
        out = [len(self.portions)]
        for p in self.portions:
            out += [len(p.tokens), p.start, p.dropped, len(p.blocks),
                    len(p.want), p.slot, *p.tokens, *p.blocks, *p.want]
        return torch.tensor(out, dtype=torch.int64)

    @classmethod
    def unflatten(cls, flat: torch.Tensor) -> "StepPlan":
        v = flat.tolist()
        at, portions = 1, []
        for _ in range(v[0]):
            n, start, dropped, nb, nw, slot = v[at:at + 6]
            at += 6
            tok, blk, want = (v[at:at + n], v[at + n:at + n + nb],
                              v[at + n + nb:at + n + nb + nw])
            at += n + nb + nw
            portions.append(Portion(tok, start, dropped, blk, want, slot))
        return cls(portions)

    # -- device tensors ------------------------------------------------------
    def build(self, block_size: int, windows, device,
              expand: bool = True) -> RaggedBatch:
        """`windows`: the distinct windows of the layers that gather the
        context of long portions; `expand` False makes every portion a short
        one."""
        P = self.portions
        short = [i for i, p in enumerate(P)
                 if not expand or len(p.tokens) <= ABSORB_MAX]
        taken = set(short)
        order = short + [i for i in range(len(P)) if i not in taken]
        n_short = len(short)

        cu = [0]
        tokens, positions, slots, first_row = [], [], [], {}
        for i in order:
            p = P[i]
            n = len(p.tokens)
            first_row[i] = cu[-1]
            cu.append(cu[-1] + n)
            tokens += p.tokens
            pos = np.arange(p.start, p.start + n)
            positions.append(pos)
            slots.append(_slots(p, pos - p.dropped, block_size))
        rows = [first_row[i] + w for i, p in enumerate(P) for w in p.want]
        seq_lens = [P[i].start - P[i].dropped + len(P[i].tokens)
                    for i in order]
        width = max(len(p.blocks) for p in P)
        tables = np.zeros((len(P), width), np.int64)
        for k, i in enumerate(order):
            tables[k, :len(P[i].blocks)] = P[i].blocks

        parts = {"tokens": tokens, "positions": np.concatenate(positions),
                 "slots": np.concatenate(slots), "cu_q": cu,
                 "seq_lens": seq_lens, "tables": tables.reshape(-1),
                 "states": [P[i].slot for i in order],
                 "seq_of": np.repeat(np.arange(len(P)), np.diff(cu)),
                 "rows": rows}
        for w in windows if n_short < len(P) else ():
            ctx, meta, at = [], [], 0
            for k, i in enumerate(order[n_short:], n_short):
                p = P[i]
                v0 = p.start - p.dropped
                lo = 0 if w is None else max(0, v0 - (w - 1))
                hi = v0 + len(p.tokens)
                ctx.append(_slots(p, np.arange(lo, hi), block_size))
                meta.append((cu[k], len(p.tokens), at, hi - lo, v0 - lo))
                at += hi - lo
            parts["ctx", w] = np.concatenate(ctx)
            parts["meta", w] = np.asarray(meta).reshape(-1)
        dev = _upload(parts, device)
        return RaggedBatch(
            tokens=dev["tokens"].long(), positions=dev["positions"],
            slots=dev["slots"], cu_q=dev["cu_q"], seq_lens=dev["seq_lens"],
            block_tables=dev["tables"].view(len(P), width),
            state_slots=dev["states"], seq_of=dev["seq_of"],
            rows=dev["rows"].long(),
            n_seqs=len(P), n_short=n_short, t_short=cu[n_short],
            max_q=max((len(P[i].tokens) for i in short), default=0),
            max_keys=max(seq_lens[:n_short], default=0),
            long_plans={w: (dev["ctx", w], dev["meta", w].view(-1, 5))
                        for w in windows if ("ctx", w) in dev},
            max_q_long=max((len(P[i].tokens) for i in order[n_short:]),
                           default=0))


def _slots(p: Portion, virtual, bs: int):
    blocks = np.asarray(p.blocks)
    return blocks[virtual // bs] * bs + virtual % bs


def _upload(parts: dict, device) -> dict:
    """Every host array in one copy; the parts are views of it."""
    arrays = {k: np.asarray(v, np.int32) for k, v in parts.items()}
    # 16-byte aligned parts
    sizes = [-(-a.size // 4) * 4 for a in arrays.values()]
    host = np.zeros(max(4, sum(sizes)), np.int32)
    at, spans = 0, {}
    for (k, a), n in zip(arrays.items(), sizes):
        host[at:at + a.size] = a
        spans[k] = (at, a.size)
        at += n
    buf = torch.from_numpy(host).to(device)
    return {k: buf[o:o + n] for k, (o, n) in spans.items()}
