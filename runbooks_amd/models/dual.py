"""Layers of models described layer by layer whose two sublayers run in
parallel, each behind a norm and an input convolution of its own
(ops/canon.py): a generalized delta rule, differential attention or latent
attention without positions beside (optionally) a PolyNorm unit, summed into
a 32-bit residual.

A layer is one kernel that adds the last layer's result, norms and convolves,
one product per sublayer, the mechanisms, which write side by side into one z,
and one product back, so the parallel sum never leaves the accumulators; its
fp32 result (or the decode GEMM's uncombined split-K slab) waits for the next
layer. `fuse()` builds the serving weights from the loaded parameters.

Tensor parallelism: heads and feed-forward columns are sharded, one all-reduce
per layer; PolyNorm's norms over all columns add one of three floats per
token. Latents, the decay's bottleneck and the input convolutions are
replicated.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import ops
from ..ops import canon as CA
from ..ops import delta as DR
from ..ops import general_delta as GD
from ..ops import latent as L
from ..ops import poly_norm as PN
from ..ops import qkv as QK
from ..ops import shared_kv as SK
from ..parallel import (ColumnParallelLinear, RowParallelLinear,
                        reduce_from_tp)
from .config import (DiffAttentionSpec, GeneralDeltaSpec, LatentAttentionSpec,
                     LayerSpec, ModelConfig, PolyNormSpec)
from .hybrid import _new_z, _project
from .streams import _local, _vector, pad


def _last_tap(n: int, taps: int, value: float, dtype):
    """Taps of a convolution that passes the current token times `value`."""
    w = torch.zeros(n, taps, dtype=dtype)
    w[:, -1] = value
    return nn.Parameter(w)


class GeneralDelta(nn.Module):
    """Generalized delta rule (one mixer)."""

    def __init__(self, cfg: ModelConfig, spec: GeneralDeltaSpec, dtype,
                 tp: int):
        super().__init__()
        D, n = cfg.hidden_size, spec.heads * spec.dim
        H = _local(spec.heads, tp, "heads")
        self.spec, self.eps = spec, cfg.norm_eps

        def col(k=D, bias=False):
            return ColumnParallelLinear(k, n, bias=bias, tp_size=tp,
                                        dtype=dtype)

        self.r_proj, self.k_proj, self.v_proj, self.g_proj = (
            col() for _ in range(4))
        self.a_proj = col(bias=True)
        self.w1_proj = ops.Linear(D, spec.decay_rank, bias=False, dtype=dtype)
        self.w2_proj = col(spec.decay_rank)
        self.o_proj = RowParallelLinear(n, D, tp_size=tp, dtype=dtype)
        self.w0 = _vector(H * spec.dim, -2, dtype)
        self.norm = ops.RMSNorm(H * spec.dim, eps=cfg.norm_eps, dtype=dtype)
        self.lay = GD.GeneralDeltaLayout(H, spec.dim, spec.vdim,
                                         spec.decay_rank)
        self.n_o = self.lay.n_o
        self.expandable = GD.general_delta_chunk_supported(self.lay, dtype)

    def fuse(self):
        lay = self.lay
        self.in_rows = GD.pack_in(lay, *(m.weight.data for m in (
            self.r_proj, self.k_proj, self.v_proj, self.a_proj, self.g_proj,
            self.w1_proj)))
        self.second_w = GD.pack_second(lay, self.w2_proj.weight.data)
        self.bias = GD.pack_bias(lay, self.w0.data, self.a_proj.bias.data)
        self.norm_w = GD.pack_norm(lay, self.norm.weight.data)
        self.out_columns = QK.pack_columns(self.o_proj.weight.data, lay.heads,
                                           lay.vdim, lay.vc)
        return [self.second_w]

    def forward(self, y, batch, state, rope, contexts, z, swz):
        lay, T = self.lay, y.shape[0]
        low = GD.tanh_rows(y, lay.off_r, lay.n_r,
                           ops.decode_ready(self.second_w, T))
        y2 = ops.fast_linear(low, self.second_w)
        o = torch.empty(T, lay.n_o, dtype=torch.float32, device=y.device)
        args = (y, y2, lay, self.bias, self.spec.decay_scale, state, batch, o)
        if batch.n_short:
            GD.general_delta_step(*args)
        if batch.n_seqs > batch.n_short:
            GD.general_delta_chunk(*args)
        DR.delta_out(o, lay, self.norm_w, y, z, self.eps, swz, y, None, batch,
                     end=lay.n_o)

    def alloc_cache(self, num_blocks, num_slots, device):
        return GD.alloc_general_delta_state(num_slots, self.lay, device)

    def block_elements(self) -> int:
        return 0

    def state_bytes(self) -> int:
        return 4 * self.lay.heads * self.lay.dc * self.lay.vc

    def covered(self) -> bool:
        return max(self.lay.dc, self.lay.vc) <= GD.MAX_DIM


class DiffAttention(nn.Module):
    """Differential attention (one mixer)."""

    def __init__(self, cfg: ModelConfig, spec: DiffAttentionSpec, dtype,
                 tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.spec, self.dtype, self.eps = spec, dtype, cfg.norm_eps
        H, G = (_local(n, tp, "heads") for n in (spec.heads, spec.kv_heads))

        def col(n):
            return ColumnParallelLinear(D, n, bias=True, tp_size=tp,
                                        dtype=dtype)

        self.q_proj = col(spec.heads * 2 * spec.dim)
        self.k_proj = col(spec.kv_heads * 2 * spec.dim)
        self.v_proj = col(spec.kv_heads * spec.vdim)
        self.o_proj = RowParallelLinear(spec.heads * spec.vdim, D, tp_size=tp,
                                        dtype=dtype)
        self.q_conv, self.k_conv, self.v_conv = (
            _last_tap(n, spec.conv, 1, dtype)
            for n in (H * 2 * spec.dim, G * 2 * spec.dim, G * spec.vdim))
        self.lq1, self.lk1, self.lq2, self.lk2 = (
            _vector(spec.dim, 0, dtype) for _ in range(4))
        self.lay = QK.QKVLayout(H, G, spec.dim, spec.vdim, maps=2)
        self.n_o = self.lay.n_z
        self.expandable = SK.shared_kv_flash_supported(self.lay, dtype)

    def fuse(self):
        lay, projs = self.lay, (self.q_proj, self.k_proj, self.v_proj)
        self.in_rows = QK.pack_qkv(lay, *(m.weight.data for m in projs))
        self.bias = QK.pack_qkv(lay, *(m.bias.data.float()[:, None]
                                       for m in projs))[:, 0].contiguous()
        self.conv_w = QK.pack_qkv(lay, *(
            c.data.float() for c in (self.q_conv, self.k_conv, self.v_conv))
        ).t().contiguous()
        lq1, lk1, lq2, lk2 = (p.data.float() for p in (
            self.lq1, self.lk1, self.lq2, self.lk2))
        factor = torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()) \
            + self.spec.diff
        self.diff = SK.DiffMaps(factor.view(1), lay.vdim, self.eps)
        self.out_columns = QK.pack_columns(self.o_proj.weight.data, lay.heads,
                                           lay.vdim, lay.vc)
        return []

    def forward(self, y, batch, cache, rope, contexts, z, swz):
        kv, tails = cache
        q = QK.qkv_conv(y, self.lay, self.bias, self.conv_w, tails, batch, kv)
        args = (q, self.lay, kv, batch, self.spec.scale, self.spec.window, z)
        kw = dict(out_scale=1.0 - self.spec.diff, diff=self.diff)
        if batch.n_short:
            SK.shared_kv_attend(*args, swz, **kw)
        if batch.n_seqs > batch.n_short:
            SK.shared_kv_flash(*args, **kw)

    def alloc_cache(self, num_blocks, num_slots, device):
        return (SK.alloc_shared_kv_cache(num_blocks, self.lay, device,
                                         self.dtype),
                QK.alloc_conv_tails(num_slots, self.spec.conv, self.lay,
                                    device, self.dtype))

    def block_elements(self) -> int:
        return self.lay.kv_heads * self.lay.ec * ops.BLOCK_SIZE

    def state_bytes(self) -> int:
        return (self.spec.conv - 1) * self.lay.n_y * \
            self.o_proj.weight.element_size()

    def covered(self) -> bool:
        return max(self.lay.hc, self.lay.vc) <= SK.MAX_HEAD


class PositionlessLatent(nn.Module):
    """Latent attention without positions (one mixer): queries come from a
    latent, too, and the gate is one number per head."""

    def __init__(self, cfg: ModelConfig, spec: LatentAttentionSpec, dtype,
                 tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.spec, self.dtype, self.eps = spec, dtype, cfg.norm_eps
        H = _local(spec.heads, tp, "heads")

        def col(n, k):
            return ColumnParallelLinear(k, n, tp_size=tp, dtype=dtype)

        def latent(n):
            return (ops.Linear(D, n, bias=False, dtype=dtype),
                    ops.RMSNorm(n, eps=cfg.norm_eps, dtype=dtype))

        self.dq_proj, self.q_norm = latent(spec.q_rank)
        self.dkv_proj, self.kv_norm = latent(spec.kv_rank)
        self.uq_proj = col(spec.heads * spec.dim, spec.q_rank)
        self.uk_proj = col(spec.heads * spec.dim, spec.kv_rank)
        self.uv_proj = col(spec.heads * spec.vdim, spec.kv_rank)
        self.g_proj = col(spec.heads, D)
        self.o_proj = RowParallelLinear(spec.heads * spec.vdim, D, tp_size=tp,
                                        dtype=dtype)
        # q stands in a tensor of its own
        self.lay = L.LatentLayout(H, spec.dim, 0, spec.vdim, spec.kv_rank, 0,
                                  own_latent=False)
        self.off_kv = ops.pad_to(spec.q_rank, 32)
        self.off_g = self.off_kv + self.lay.ec
        self.n_o = self.lay.off_act
        self.expandable = (L.latent_flash_supported(self.lay, dtype) and
                           dtype == torch.bfloat16)

    def fuse(self):
        lay, s = self.lay, self.spec
        self.in_rows = torch.cat([
            pad(w.data, (0, 0, 0, n - w.shape[0])) for w, n in (
                (self.dq_proj.weight, self.off_kv),
                (self.dkv_proj.weight, lay.ec),
                (self.g_proj.weight, ops.pad_to(lay.heads, 8)))])
        uq = L._pad_rows(self.uq_proj.weight.data, lay.heads, (lay.dim,),
                         (lay.dimc,))
        self.q_w = pad(uq, (0, self.off_kv - s.q_rank,
                            0, -uq.shape[0] % 32)).contiguous()
        self.norms = ((0, self.off_kv), (s.q_rank, s.kv_rank),
                      (self.q_norm.weight.data.float(),
                       self.kv_norm.weight.data.float()))
        uk, uv = self.uk_proj.weight.data, self.uv_proj.weight.data
        r = lay.rc - lay.rank
        self.absorb_w = L.pack_heads(pad(
            uk.view(lay.heads, lay.dim, -1), (0, r, 0, lay.dimc - lay.dim)))
        self.expand_w = L.pack_heads(pad(
            uv.view(lay.heads, lay.vdim, -1), (0, r, 0, lay.vc - lay.vdim)
        ).transpose(1, 2))
        self.context_w = L.pack_expand(lay, uk, uv)
        self.out_columns = QK.pack_columns(self.o_proj.weight.data, lay.heads,
                                           lay.vdim, lay.vc)
        return [self.q_w]

    def forward(self, y, batch, cache, rope, contexts, z, swz):
        lay, spec = self.lay, self.spec
        ready = ops.decode_ready(self.q_w, y.shape[0])
        c = L.latent_norms(
            y, self.norms, self.eps, batch.slots, cache,
            ops.decode_operand(y.shape[0], self.off_kv, y) if ready else None)
        q = ops.fast_linear(c, self.q_w)
        gate = dict(off_g=self.off_g, head_gate=True)
        if batch.t_short:
            q_lat = L.latent_absorb(q, lay, self.absorb_w, batch.t_short)
            o_lat = L.latent_attend(q_lat, q, lay, cache, batch, spec.scale,
                                    None)
            L.latent_expand(o_lat, lay, self.expand_w, y, z, swz, **gate)
        if batch.long_plans:
            slots, meta = batch.long_plans[None]
            ctx = cache.view(-1, lay.ec).index_select(0, slots)
            kv = nn.functional.linear(ctx, self.context_w)
            L.latent_flash(q, lay, kv, ctx, meta, batch.max_q_long,
                           spec.scale, None, z, y, **gate)

    def alloc_cache(self, num_blocks, num_slots, device):
        return ops.alloc_latent_cache(num_blocks, self.lay, device,
                                      self.dtype)

    def block_elements(self) -> int:
        return self.lay.ec * ops.BLOCK_SIZE

    def state_bytes(self) -> int:
        return 0

    def covered(self) -> bool:
        return self.lay.ec <= L.MAX_ROW


class PolyUnit(nn.Module):
    """down(PolyNorm(up))."""

    def __init__(self, cfg: ModelConfig, spec: PolyNormSpec, dtype, tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.ff, self.total, self.tp = (_local(spec.ff, tp, "columns"),
                                        spec.ff, tp)
        self.eps = cfg.norm_eps
        self.up_proj = ColumnParallelLinear(D, spec.ff, tp_size=tp,
                                            dtype=dtype)
        self.down_proj = RowParallelLinear(spec.ff, D, tp_size=tp,
                                           dtype=dtype)
        act = torch.zeros(4, dtype=dtype)
        act[0] = 1
        self.act = nn.Parameter(act)

    def fuse(self):
        self.in_rows = self.up_proj.weight.data
        self.act_v = self.act.data.float()

    def forward(self, u, z, off: int, swz):
        sums = None
        if self.tp > 1:
            sums = reduce_from_tp(PN.power_sums(u, self.ff))
        PN.poly_norm(u, self.ff, self.total, self.act_v, self.eps, z, off,
                     swz, sums)


class DualBlock(nn.Module):
    def __init__(self, cfg: ModelConfig, spec: LayerSpec, dtype, tp: int):
        super().__init__()
        self.spec, self.tp, self.dtype = spec, tp, dtype
        self.eps, self.taps = cfg.norm_eps, cfg.canon
        self.width = cfg.hidden_size
        kind = {GeneralDeltaSpec: GeneralDelta,
                DiffAttentionSpec: DiffAttention,
                LatentAttentionSpec: PositionlessLatent}[type(spec.mixer)]
        self.mixer = kind(cfg, spec.mixer, dtype, tp)
        self.mlp = (PolyUnit(cfg, spec.mlp, dtype, tp) if spec.mlp else None)
        self.parts = [self.mixer] + ([self.mlp] if spec.mlp else [])
        for i in range(1, len(self.parts) + 1):
            setattr(self, f"norm{i}", ops.RMSNorm(
                self.width, eps=cfg.norm_eps, dtype=dtype,
                offset=cfg.norm_offset))
            setattr(self, f"canon{i}", _last_tap(self.width, self.taps, 0,
                                                 dtype))
        off, ff = self.mixer.n_o, self.mlp.ff if spec.mlp else 0
        self.n_z = ops.pad_to(off + ops.pad_to(ff, 8), 32)

    @property
    def expandable(self) -> bool:
        return self.mixer.expandable

    @torch.no_grad()
    def fuse(self) -> list[torch.Tensor]:
        """Serving weights from the loaded parameters; returns those the
        decode GEMM may keep a copy of."""
        weights = list(self.mixer.fuse())
        if self.mlp is not None:
            self.mlp.fuse()
        D = self.width
        for p in self.parts:
            rows = p.in_rows
            p.in_w = pad(rows, (0, -D % 32, 0, -rows.shape[0] % 32)
                         ).contiguous()
            del p.in_rows
        out = [self.mixer.out_columns]
        del self.mixer.out_columns
        if self.mlp is not None:
            up = self.mlp.up_proj
            up.weight = nn.Parameter(self.mlp.in_w[:self.mlp.ff, :D],
                                     requires_grad=False)
            out.append(self.mlp.down_proj.weight.data)
        out = torch.cat(out, dim=1)
        self.out_w = pad(out, (0, self.n_z - out.shape[1])).contiguous()
        n = range(1, len(self.parts) + 1)
        norms = [getattr(self, f"norm{i}") for i in n]
        self.coef = CA.pack_coefficients(
            [m.offset + m.weight.data.float() for m in norms],
            [getattr(self, f"canon{i}").data for i in n])
        return weights + [p.in_w for p in self.parts] + [self.out_w]

    def step(self, x, delta, batch, cache, rope, contexts):
        """x [T, D] fp32 residual before this layer without `delta`, the
        last layer's pending output; adds delta to x in place and returns
        this layer's own pending output."""
        T, (kept, tails) = x.shape[0], cache
        hs = CA.canon_norm(x, delta, self.coef, tails, batch, self.eps,
                           self.dtype, [ops.decode_ready(p.in_w, T)
                                        for p in self.parts])
        y, *u = (ops.fast_linear(h, p.in_w) for h, p in zip(hs, self.parts))
        z, swz = _new_z(self, y, self.out_w,
                        filled=bool(u) or self.n_z == self.mixer.n_o)
        self.mixer(y, batch, kept, rope, contexts, z, swz)
        if u:
            self.mlp(u[0], z, self.mixer.n_o, swz)
        return _project(z, self.out_w, self.tp)

    def alloc_cache(self, num_blocks: int, num_slots: int, device):
        return (self.mixer.alloc_cache(num_blocks, num_slots, device),
                CA.alloc_canon_tails(num_slots, self.taps, self.width,
                                     device))

    def block_elements(self) -> int:
        return self.mixer.block_elements()

    def state_bytes(self) -> int:
        return self.mixer.state_bytes() + 4 * (self.taps - 1) * self.width

    def covered(self) -> bool:
        """The kernels run these sizes."""
        return self.mixer.covered()
