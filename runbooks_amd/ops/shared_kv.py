"""Attention in which a token's unrotated key doubles as its value, over a
paged cache.

Around one projection `y` and one output projection that reads `z`:

    y = [ q heads | k heads ],   z = [ heads of the result ]

  * ``shared_kv_prep``    rotates q in y and writes the cached rows
  * ``shared_kv_attend``  attention of decoded tokens and short portions
  * ``shared_kv_flash``   the same attention for long portions

A head of q and k has the rotated dimensions first, then the others, each
part padded to a multiple of 8 with zero rows of the packed weight. The
cache keeps, per token and kv head, the key as the scores need it and after
it once more only the rotated dimensions as they were before rotation:

    [ rotated | others | unrotated ]     key = the first hc columns,
                                         value = the last hc columns

so a row has dim + rotated elements, not 2 dim. The value's columns come in
the order [others | unrotated]; pack_out puts W_o's columns in that order.

GPU tensors run csrc/shared_kv_*.hip; CPU tensors the plain references here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .kvcache import BLOCK_SIZE
from .latent import pad_to


MAX_HEAD = 1024                # padded head size the kernels run


@dataclass(frozen=True)
class SharedKVLayout:
    """Columns of y, z and the cache rows of one layer (sizes local to this
    rank)."""
    heads: int
    kv_heads: int
    dim: int
    rot: int                   # rotated dimensions

    @property
    def group(self):
        return self.heads // self.kv_heads

    @property
    def rotc(self):
        return pad_to(self.rot, 8)

    @property
    def hc(self):              # one head
        return self.rotc + pad_to(self.dim - self.rot, 8)

    @property
    def ec(self):              # one cached row
        return self.rotc + self.hc

    @property
    def voff(self):            # first column of the value in a row
        return self.rotc

    @property
    def off_k(self):
        return self.heads * self.hc

    @property
    def n_y(self):
        return pad_to((self.heads + self.kv_heads) * self.hc, 32)

    @property
    def n_z(self):
        return pad_to(self.heads * self.hc, 16)


def alloc_shared_kv_cache(num_blocks: int, lay: SharedKVLayout, device,
                          dtype=torch.bfloat16):
    """[blocks, kv heads, tokens, row]; the padding stays zero."""
    return torch.zeros(num_blocks, lay.kv_heads, BLOCK_SIZE, lay.ec,
                       device=device, dtype=dtype)


# ---------------------------------------------------------------------------
# weights
# ---------------------------------------------------------------------------

def pack_in(lay: SharedKVLayout, q, k):
    """Rows of the joint q and k projection, in y's layout."""
    w = torch.cat([q, k]).view(-1, lay.dim, q.shape[1])
    out = w.new_zeros(w.shape[0], lay.hc, w.shape[2])
    out[:, :lay.rot] = w[:, :lay.rot]
    out[:, lay.rotc:lay.rotc + lay.dim - lay.rot] = w[:, lay.rot:]
    out = out.view(-1, w.shape[2])
    return torch.nn.functional.pad(
        out, (0, 0, 0, lay.n_y - out.shape[0])).contiguous()


def pack_out(lay: SharedKVLayout, o):
    """Columns of the output projection, in z's layout (a head's unrotated
    part first)."""
    rest = lay.dim - lay.rot
    w = o.new_zeros(o.shape[0], lay.n_z)
    heads = w[:, :lay.heads * lay.hc].view(-1, lay.heads, lay.hc)
    src = o.view(-1, lay.heads, lay.dim)
    heads[:, :, :rest] = src[:, :, lay.rot:]
    at = lay.hc - lay.rotc
    heads[:, :, at:at + lay.rot] = src[:, :, :lay.rot]
    return w


# ---------------------------------------------------------------------------
# references (CPU)
# ---------------------------------------------------------------------------

def rotate_halves_ref(x, cos, sin, positions):
    """x [T, ..., d], tables [positions, dims/2]: dimension i turns with
    i + dims/2, dimensions from `dims` on pass. Returns fp32."""
    half = cos.shape[1]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [half]
    c = cos[positions.long()].view(shape)
    s = sin[positions.long()].view(shape)
    out = x.float().clone()
    u, v = x[..., :half].float(), x[..., half:2 * half].float()
    out[..., :half] = u * c - v * s
    out[..., half:2 * half] = v * c + u * s
    return out


def _prep_ref(y, lay, cos, sin, positions, slots, cache):
    T = y.shape[0]
    q = y[:, :lay.off_k].view(T, lay.heads, lay.hc)
    k = y[:, lay.off_k:lay.off_k + lay.kv_heads * lay.hc].reshape(
        T, lay.kv_heads, lay.hc)
    s = slots.long()
    rows = torch.cat([rotate_halves_ref(k, cos, sin, positions),
                      k[..., :lay.rotc].float()], dim=-1)
    cache[s // BLOCK_SIZE, :, s % BLOCK_SIZE] = rows.to(cache.dtype)
    q.copy_(rotate_halves_ref(q, cos, sin, positions))


def visible_ref(qpos, kpos, window, chunk=None, dropped=0):
    """[queries, keys]: the keys a query sees, of its window or its chunk
    (absolute position = retained position + dropped)."""
    seen = kpos[None] <= qpos[:, None]
    if window is not None:
        seen = seen & (kpos[None] > qpos[:, None] - window)
    if chunk is not None:
        seen = seen & ((kpos + dropped)[None] // chunk ==
                       (qpos + dropped)[:, None] // chunk)
    return seen


@dataclass(frozen=True)
class DiffMaps:
    """Two attention maps per head, the second one's result subtracted:
    rms_norm(o1 - factor o2) per head."""
    factor: torch.Tensor       # [1] fp32
    vdim: int                  # columns the norm counts
    eps: float


def _attend_ref(y, lay, cache, batch, seqs, scale, window, z, chunk=None,
                sink=None, out_scale=1.0, diff=None):
    maps = 1 if diff is None else 2
    for b in seqs:
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        n = int(batch.seq_lens[b])
        pos = torch.arange(n)
        blk = batch.block_tables[b].long()[pos // BLOCK_SIZE]
        rows = cache[blk, :, pos % BLOCK_SIZE].float()     # [n, G, ec]
        # group members are heads, or (head, map) pairs
        q = y[t0:t1, :lay.off_k].float().view(
            t1 - t0, lay.kv_heads, lay.group, maps, lay.hc)
        k = rows[..., :maps * lay.hc].view(n, lay.kv_heads, maps, lay.hc)
        s = torch.einsum("qgrmd,kgmd->grmqk", q, k).flatten(1, 2) * scale
        dropped = int(batch.positions[t0]) - (n - (t1 - t0))
        hidden = ~visible_ref(pos[n - (t1 - t0):], pos, window, chunk,
                              dropped)
        s = s.masked_fill(hidden, float("-inf"))
        if sink is not None:      # one more entry of the denominator
            extra = sink.view(lay.kv_heads, lay.group, 1, 1).expand(
                *s.shape[:-1], 1)
            s = torch.cat([s, extra], dim=-1)
        p = torch.softmax(s, dim=-1)[..., :n]
        o = torch.einsum("grqk,kgd->qgrd", p, rows[..., lay.voff:])
        if diff is not None:
            o = o[:, :, 0::2] - diff.factor * o[:, :, 1::2]
            o = o * torch.rsqrt(o.pow(2).sum(-1, keepdim=True) / diff.vdim +
                                diff.eps)
        o = (o * out_scale).reshape(t1 - t0, -1)
        z[t0:t1, :o.shape[1]] = o.to(z.dtype)


# ---------------------------------------------------------------------------
# ops
# ---------------------------------------------------------------------------

def shared_kv_prep(y, lay, cos, sin, positions, slots, cache):
    """Rotate q inside y and write the keys' rows to `cache` at `slots`."""
    if not _backend.use_hip(y):
        return _prep_ref(y, lay, cos, sin, positions, slots, cache)
    _backend.ext().shared_kv_prep(y, cos, sin, positions, slots, cache,
                                  lay.heads, lay.rotc)


def attend_split(n_seqs: int, workgroups: int, max_keys: int | None,
                 window: int | None, max_q: int) -> int:
    """Cache splits per workgroup of 16 query rows: about four workgroups
    per CU, each with at least 256 keys."""
    keys = max_keys
    if window is not None:
        w = window + max_q - 1
        keys = w if keys is None else min(keys, w)
    fill = max(1, 1024 // max(1, n_seqs * workgroups))
    if keys is not None:
        fill = min(fill, -(-keys // 256))
    return max(1, min(32, fill))


def shared_kv_attend(y, lay, cache, batch, scale, window, z, swz=None,
                     chunk=None, sink=None, out_scale=1.0, diff=None):
    """z's first t_short rows: attention of the batch's short portions. A
    query at retained position i sees keys j with 0 <= i - j < window, or
    those up to its own of its chunk. `sink` [heads] fp32: one more entry of
    the softmax's denominator. The result is multiplied by out_scale. With
    `diff` (DiffMaps) every head has two queries, the kv heads' rows two keys,
    [ key | key | value ]."""
    if not _backend.use_hip(y):
        return _attend_ref(y, lay, cache, batch, range(batch.n_short), scale,
                           window, z, chunk, sink, out_scale, diff)
    maps = 1 if diff is None else 2
    tiles = -(-batch.max_q * lay.group * maps // 16) * lay.kv_heads
    nsplit = attend_split(batch.n_short, tiles, batch.max_keys,
                          window or chunk, batch.max_q)
    _backend.ext().shared_kv_attend(
        y, cache, batch.block_tables, batch.cu_q, batch.seq_lens,
        batch.n_short, batch.t_short, batch.max_q, nsplit, scale, window or 0,
        lay.heads, lay.hc, lay.voff, z, swz, chunk or 0, batch.positions,
        sink, out_scale, *_diff_args(diff))


def _diff_args(diff):
    return (None, 0, 0.0) if diff is None else (diff.factor, diff.vdim,
                                                diff.eps)


def shared_kv_flash_supported(lay: SharedKVLayout, dtype) -> bool:
    return dtype == torch.bfloat16 and max(lay.hc, lay.ec - lay.voff) <= 256


def shared_kv_flash(y, lay, cache, batch, scale, window, z, chunk=None,
                    sink=None, out_scale=1.0, diff=None):
    """z's other rows: the same attention for the long portions."""
    n = batch.n_seqs - batch.n_short
    if not _backend.use_hip(y):
        return _attend_ref(y, lay, cache, batch,
                           range(batch.n_short, batch.n_seqs), scale, window,
                           z, chunk, sink, out_scale, diff)
    _backend.ext().shared_kv_flash(
        y, cache, batch.block_tables, batch.cu_q, batch.seq_lens,
        batch.n_short, n, batch.max_q_long, scale, window or 0, lay.heads,
        lay.hc, lay.voff, z, chunk or 0, batch.positions, sink, out_scale,
        *_diff_args(diff))
