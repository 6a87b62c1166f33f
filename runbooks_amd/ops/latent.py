"""Latent attention: one cached latent (and one rotated key part) per token.

The ops of a layer whose sublayers share one normed input, around one wide
projection `y` and one output projection that reads `z`:

    y = [ q | latent, rotated key | gate of the heads | mlp gate | mlp up ]
    z = [ gated heads | mlp activation ]

  * ``latent_prep``    rotates q in y, norms/rotates the latent row and
                       writes it to the paged cache, and fills z's mlp part
  * ``latent_absorb``  q -> latent space (per head, W_uk transposed)
  * ``latent_attend``  attention over the cached latents (any portion)
  * ``latent_expand``  latent -> value space (W_uv) times the output gate
  * ``latent_flash``   the same attention for long portions, on keys and
                       values expanded from the context's latents

Without a rotated part and with queries from a latent of their own,

    y = [ query latent | latent | gates ],   q = product of the former

``latent_norms`` takes the place of latent_prep: it norms both latents; the
other ops then read q in a tensor of its own. The output gate is one number
per value column, or (head_gate) one per head.

Every per-head or per-section size is padded to a multiple of 8 elements
inside y, z, the cache and the packed weights (zero rows), so the kernels
read 16 bytes per lane for any model size.

GPU tensors run csrc/latent_*.hip; CPU tensors the plain references here.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _backend
from .kvcache import BLOCK_SIZE


MAX_ROW = 2048                 # elements of a cache row the kernels run


def pad_to(n: int, m: int) -> int:
    return -(-n // m) * m


@dataclass(frozen=True)
class LatentLayout:
    """Column layout of y, z and the cache rows of one layer (sizes local
    to this rank)."""
    heads: int
    dim: int
    rot: int
    vdim: int
    rank: int
    ff: int
    own_latent: bool           # this layer projects latents of its own

    @property
    def dimc(self):
        return pad_to(self.dim, 8)

    @property
    def rotc(self):
        return pad_to(self.rot, 8)

    @property
    def qc(self):              # one head of q
        return self.dimc + self.rotc

    @property
    def vc(self):
        return pad_to(self.vdim, 8)

    @property
    def rc(self):
        return pad_to(self.rank, 8)

    @property
    def ec(self):              # one cache row
        return self.rc + self.rotc

    @property
    def fc(self):
        return pad_to(self.ff, 8)

    @property
    def off_kv(self):
        return self.heads * self.qc

    @property
    def off_g(self):
        return self.off_kv + (self.ec if self.own_latent else 0)

    @property
    def off_gate(self):
        return self.off_g + self.heads * self.vc

    @property
    def off_up(self):
        return self.off_gate + self.fc

    @property
    def n_y(self):
        return pad_to(self.off_up + self.fc, 32)

    @property
    def off_act(self):
        return self.heads * self.vc

    @property
    def n_z(self):
        return pad_to(self.off_act + self.fc, 16)


def alloc_latent_cache(num_blocks: int, lay: LatentLayout, device,
                       dtype=torch.bfloat16, block_size: int = BLOCK_SIZE):
    """[blocks, tokens, latent | rotated key]; the padding stays zero."""
    return torch.zeros(num_blocks, block_size, lay.ec, device=device,
                       dtype=dtype)


# ---------------------------------------------------------------------------
# weights
# ---------------------------------------------------------------------------

def _pad_rows(w, groups, sizes, padded):
    """[groups * sum(sizes), K] -> [groups * sum(padded), K]: each part of
    each group gets zero rows up to its padded size."""
    K = w.shape[1]
    w = w.view(groups, sum(sizes), K)
    out = w.new_zeros(groups, sum(padded), K)
    a = b = 0
    for s, p in zip(sizes, padded):
        out[:, b:b + s] = w[:, a:a + s]
        a, b = a + s, b + p
    return out.view(-1, K)


def pack_wide(lay: LatentLayout, q, dkv, g, gate, up):
    """Rows of the wide projection, in y's layout."""
    parts = [_pad_rows(q, lay.heads, (lay.dim, lay.rot),
                       (lay.dimc, lay.rotc))]
    if lay.own_latent:
        parts.append(_pad_rows(dkv, 1, (lay.rank, lay.rot),
                               (lay.rc, lay.rotc)))
    parts.append(_pad_rows(g, lay.heads, (lay.vdim,), (lay.vc,)))
    if lay.ff:
        parts += [_pad_rows(w, 1, (lay.ff,), (lay.fc,)) for w in (gate, up)]
    w = torch.cat(parts)
    if w.shape[0] < lay.n_y:
        w = torch.cat([w, w.new_zeros(lay.n_y - w.shape[0], w.shape[1])])
    return w.contiguous()


def pack_out(lay: LatentLayout, o, down):
    """Columns of the output projection, in z's layout."""
    w = o.new_zeros(o.shape[0], lay.n_z)
    w[:, :lay.off_act].view(-1, lay.heads, lay.vc)[:, :, :lay.vdim] = \
        o.view(-1, lay.heads, lay.vdim)
    if lay.ff:
        w[:, lay.off_act:lay.off_act + lay.ff] = down
    return w


def pack_expand(lay: LatentLayout, uk, uv):
    """[H * (dimc + vc), rc]: unrotated keys and values of all heads as one
    product of the latents."""
    w = torch.cat([uk.view(lay.heads, lay.dim, -1),
                   uv.view(lay.heads, lay.vdim, -1)], dim=1)
    w = _pad_rows(w.reshape(-1, w.shape[-1]), lay.heads,
                  (lay.dim, lay.vdim), (lay.dimc, lay.vc))
    return torch.nn.functional.pad(w, (0, lay.rc - lay.rank)).contiguous()


def pack_heads(w):
    """Per-head matrices [H, K, N] (y_h = x_h @ w_h) in the layout
    `head_gemm` reads: bf16 GPU weights in MFMA fragment order
    [H, N/16, K/32, 64 lanes, 8], others as they are."""
    if not (w.is_cuda and w.dtype == torch.bfloat16):
        return w.contiguous()
    H, K, N = w.shape
    w = torch.nn.functional.pad(w, (0, pad_to(N, 16) - N,
                                    0, pad_to(K, 32) - K))
    # lane = 16 * (k / 8 % 4) + n % 16, element = k % 8
    return (w.view(H, w.shape[1] // 32, 4, 8, w.shape[2] // 16, 16)
            .permute(0, 4, 1, 2, 5, 3).contiguous())


# ---------------------------------------------------------------------------
# references (CPU)
# ---------------------------------------------------------------------------

def rope_interleaved_ref(x, cos, sin, positions):
    """x [T, ..., d], tables [positions, dims/2]: pairs (2i, 2i+1) of the
    first `dims` dimensions turn, the rest pass. Returns fp32."""
    half = cos.shape[1]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [half]
    c = cos[positions.long()].view(shape)
    s = sin[positions.long()].view(shape)
    out = x.float().clone()
    u, v = x[..., 0:2 * half:2].float(), x[..., 1:2 * half:2].float()
    out[..., 0:2 * half:2] = u * c - v * s
    out[..., 1:2 * half:2] = v * c + u * s
    return out


def clamped_glu_ref(g, u, limit, alpha, shift):
    g = g.float().clamp(max=limit)
    u = u.float().clamp(-limit, limit)
    return g * torch.sigmoid(alpha * g) * (u + shift)


def _prep_ref(y, lay, cos, sin, positions, slots, cache, w, eps, mlp, z):
    T = y.shape[0]
    q = y[:, :lay.off_kv].view(T, lay.heads, lay.qc)
    q[..., lay.dimc:] = rope_interleaved_ref(
        q[..., lay.dimc:], cos, sin, positions).to(y.dtype)
    if lay.own_latent:
        kv = y[:, lay.off_kv:lay.off_g].float()
        c = kv[:, :lay.rank]
        c = c * torch.rsqrt(c.pow(2).mean(-1, keepdim=True) + eps) * w.float()
        flat = cache.view(-1, lay.ec)
        s = slots.long()
        flat[s, :lay.rank] = c.to(cache.dtype)
        flat[s, lay.rc:] = rope_interleaved_ref(
            kv[:, lay.rc:], cos, sin, positions).to(cache.dtype)
    z[:, lay.off_act:] = 0
    if lay.ff:
        z[:, lay.off_act:lay.off_act + lay.fc] = clamped_glu_ref(
            y[:, lay.off_gate:lay.off_up],
            y[:, lay.off_up:lay.off_up + lay.fc],
            mlp.limit, mlp.alpha, mlp.shift).to(z.dtype)


def _masked_softmax_ref(s, qpos, kpos, window):
    """s [..., q, k]; positions [q], [k]."""
    d = qpos[:, None] - kpos[None, :]
    ok = d >= 0
    if window is not None:
        ok &= d < window
    return torch.softmax(s.masked_fill(~ok, float("-inf")), dim=-1)


def _attend_ref(q_lat, y, lay, cache, batch, scale, window):
    out = torch.zeros_like(q_lat)
    rows = cache.view(-1, lay.ec)
    for b in range(batch.n_short):
        t0, t1 = int(batch.cu_q[b]), int(batch.cu_q[b + 1])
        n = int(batch.seq_lens[b])
        pos = torch.arange(n)
        slot = batch.block_tables[b].long()[pos // BLOCK_SIZE] * BLOCK_SIZE \
            + pos % BLOCK_SIZE
        kv = rows[slot].float()
        q = torch.cat([q_lat[t0:t1].float(),
                       y[t0:t1, :lay.off_kv].view(
                           t1 - t0, lay.heads, lay.qc)[..., lay.dimc:]
                       .float()], dim=-1)
        s = torch.einsum("qhe,ke->hqk", q, kv) * scale
        p = _masked_softmax_ref(s, pos[n - (t1 - t0):], pos, window)
        out[t0:t1] = torch.einsum("hqk,kr->qhr", p,
                                  kv[:, :lay.rc]).to(out.dtype)
    return out


def gated_ref(o, lay, gate, off, head_gate):
    """o [T, H, vc] times the sigmoid gates in `gate`'s columns from off."""
    T = o.shape[0]
    if head_gate:
        g = gate[:, off:off + lay.heads].float()[..., None]
    else:
        g = gate[:, off:off + lay.heads * lay.vc].float().view(o.shape)
    return (o * torch.sigmoid(g)).reshape(T, -1)


def _flash_ref(y, lay, kv, ctx, meta, scale, window, z, gate, off_g,
               head_gate):
    for q0, nq, k0, nk, rel in meta.tolist():
        q = y[q0:q0 + nq, :lay.off_kv].view(nq, lay.heads, lay.qc).float()
        e = kv[k0:k0 + nk].view(nk, lay.heads, lay.dimc + lay.vc).float()
        kr = ctx[k0:k0 + nk, lay.rc:].float()
        s = (torch.einsum("qhd,khd->hqk", q[..., :lay.dimc],
                          e[..., :lay.dimc]) +
             torch.einsum("qhd,kd->hqk", q[..., lay.dimc:], kr)) * scale
        p = _masked_softmax_ref(s, torch.arange(nq) + rel, torch.arange(nk),
                                window)
        o = torch.einsum("hqk,khv->qhv", p, e[..., lay.dimc:])
        z[q0:q0 + nq, :lay.off_act] = gated_ref(
            o, lay, gate[q0:q0 + nq], off_g, head_gate).to(z.dtype)


# ---------------------------------------------------------------------------
# ops
# ---------------------------------------------------------------------------

def latent_prep(y, lay, cos, sin, positions, slots, cache, norm_w, eps, mlp,
                z, swz=None):
    """Rotate q inside y; for a layer with latents of its own write the
    normed latent and the rotated key to `cache` at `slots`; fill z's mlp
    part (and, when given, the same part of the decode-GEMM operand
    `swz`)."""
    if not _backend.use_hip(y):
        return _prep_ref(y, lay, cos, sin, positions, slots, cache, norm_w,
                         eps, mlp, z)
    limit, alpha, shift = ((mlp.limit, mlp.alpha, mlp.shift) if mlp
                           else (0.0, 0.0, 0.0))
    _backend.ext().latent_prep(
        y, cos, sin, positions, slots, cache if lay.own_latent else None,
        norm_w if lay.own_latent else None, z, swz, lay.heads, lay.dimc,
        lay.rotc, lay.rank, lay.rc, lay.off_kv, lay.off_gate, lay.off_up,
        lay.fc, lay.off_act, eps, limit, alpha, shift)


def latent_norms(y, parts, eps, slots, cache, swz=None):
    """RMS norms of both latents in y. parts: (first columns, sizes, weights
    fp32) of the query latent and of the cached one, as three pairs. Returns
    the former, [T, its size padded to 32]; the latter goes to `cache` at
    `slots`."""
    (oq, oc), (nq, nc), (wq, wc) = parts
    out = torch.empty(y.shape[0], pad_to(nq, 32), dtype=y.dtype,
                      device=y.device)
    if not _backend.use_hip(y):
        def norm(at, n, w):
            c = y[:, at:at + n].float()
            return (c * torch.rsqrt(c.pow(2).mean(-1, keepdim=True) + eps) *
                    w).to(y.dtype)
        out.zero_()
        out[:, :nq] = norm(oq, nq, wq)
        cache.view(-1, cache.shape[-1])[slots.long(), :nc] = norm(oc, nc, wc)
        return out
    _backend.ext().latent_norms(y, oq, nq, wq, out, swz, oc, nc, wc, cache,
                                slots, eps)
    if swz is not None:
        out._rb_swz = swz
    return out


def latent_absorb(y, lay, w_absorb, T):
    """First T rows of q, unrotated part, into latent space:
    [T, heads, rc]."""
    if not _backend.use_hip(y):
        q = y[:T, :lay.off_kv].view(T, lay.heads, lay.qc)[..., :lay.dimc]
        return torch.einsum("thd,hdr->thr", q.float(),
                            w_absorb.float()).to(y.dtype)
    out = torch.empty(T, lay.heads, lay.rc, dtype=y.dtype, device=y.device)
    _backend.ext().head_gemm(
        y, 0, lay.qc, w_absorb, lay.dimc, lay.rc, out.view(T, -1), 0, lay.rc,
        None, 0, None, T, lay.heads, False)
    return out


def latent_expand(o_lat, lay, w_expand, gate, z, swz=None, off_g=None,
                  head_gate=False):
    """z's head part of the first rows: value-space heads times the sigmoid
    output gates, in columns of `gate` from off_g (None: as y has them)."""
    T = o_lat.shape[0]
    off_g = lay.off_g if off_g is None else off_g
    if not _backend.use_hip(o_lat):
        o = torch.einsum("thr,hrv->thv", o_lat.float(), w_expand.float())
        z[:T, :lay.off_act] = gated_ref(o, lay, gate[:T], off_g,
                                        head_gate).to(z.dtype)
        return
    _backend.ext().head_gemm(
        o_lat.view(T, -1), 0, lay.rc, w_expand, lay.rc, lay.vc, z, 0, lay.vc,
        gate, off_g, swz, T, lay.heads, head_gate)


def attend_split(n_seqs: int, row_tiles: int, max_keys: int | None,
                 window: int | None, max_q: int) -> int:
    """Cache splits per (sequence, row tile): one workgroup per CU, each
    with at least two 64-key tiles."""
    keys = max_keys
    if window is not None:
        w = window + max_q - 1
        keys = w if keys is None else min(keys, w)
    base = max(1, n_seqs * row_tiles)
    fill = max(1, -(-256 // base))
    if keys is not None:
        fill = min(fill, -(-keys // 128))
    return max(1, min(32, fill))


def latent_attend(q_lat, y, lay, cache, batch, scale, window):
    """Attention of the batch's short portions over the cached latents:
    [t_short, heads, rc]. A query at retained position i sees keys j with
    0 <= i - j < window."""
    if not _backend.use_hip(y):
        return _attend_ref(q_lat, y, lay, cache, batch, scale, window)
    ext = _backend.ext()
    rows = batch.max_q * lay.heads
    tiles = -(-rows // ext.latent_attend_rows(rows, lay.rc, lay.rotc,
                                              y.dtype == torch.bfloat16))
    nsplit = attend_split(batch.n_short, tiles, batch.max_keys, window,
                          batch.max_q)
    return ext.latent_attend(
        q_lat, y, lay.dimc, lay.qc, cache, batch.block_tables, batch.cu_q,
        batch.seq_lens, batch.n_short, batch.max_q, nsplit, scale,
        window or 0, lay.rc)


def latent_flash_supported(lay: LatentLayout, dtype) -> bool:
    return lay.dimc + lay.rotc <= 256 and lay.vc <= 256


def latent_flash(y, lay, kv, ctx, meta, max_q, scale, window, z, gate=None,
                 off_g=None, head_gate=False):
    """z's head part of the long portions. kv [Tk, H, dimc + vc]: keys and
    values expanded from the context rows `ctx` [Tk, ec]; meta rows as in
    RaggedBatch.long_plans; gates as in latent_expand (None: in y)."""
    gate = y if gate is None else gate
    off_g = lay.off_g if off_g is None else off_g
    if not _backend.use_hip(y):
        return _flash_ref(y, lay, kv, ctx, meta, scale, window, z, gate,
                          off_g, head_gate)
    _backend.ext().latent_flash(y, kv, ctx, meta, z, lay.heads, lay.dimc,
                                lay.rotc, lay.vc, lay.rc, gate, off_g,
                                head_gate, max_q, scale, window or 0)
