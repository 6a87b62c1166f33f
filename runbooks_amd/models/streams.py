"""Layers of models described layer by layer whose residual is several
streams with learned mixing (ops/streams.py): a gated delta rule, or chunked
attention beside a minGRU, then (optionally) a squared-ReLU unit or a mixture
of them.

A sublayer is one product of its normed input (projections and, as further
rows, the gate of its result), the mechanism, and one product back, whose
fp32 result (or the decode GEMM's uncombined split-K slab) waits as a
`Pending` for the norm that follows it. `fuse()` builds the serving weights
from the loaded parameters.

Tensor parallelism: heads, the minGRU's width and the columns of every
feed-forward are sharded, one all-reduce per sublayer; gates of results,
bottlenecks and routers are replicated.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import ops
from ..ops import delta as DR
from ..ops import min_gru as MG
from ..ops import moe as ME
from ..ops import qkv as QK
from ..ops import shared_kv as SK
from ..ops import streams as ST
from ..parallel import (ColumnParallelLinear, RowParallelLinear,
                        reduce_from_tp)
from .config import (AttentionSpec, GatedDeltaSpec, LayerSpec, MinGRUSpec,
                     ModelConfig, MoESpec, SquaredReluSpec, TwinSpec)
from .hybrid import _new_z, _project

pad = nn.functional.pad


def _local(n: int, tp: int, what: str) -> int:
    if n % tp:
        raise ValueError(f"{n} {what} do not divide tp={tp}")
    return n // tp


def _vector(n, value, dtype):
    return nn.Parameter(torch.full(n if isinstance(n, tuple) else (n,),
                                   float(value), dtype=dtype))


class GatedDelta(nn.Module):
    """Gated delta rule (one mixer)."""

    def __init__(self, cfg: ModelConfig, spec: GatedDeltaSpec, dtype,
                 tp: int):
        super().__init__()
        D, d, e = cfg.hidden_size, spec.dim, spec.vdim
        H, G = (_local(n, tp, "heads") for n in (spec.heads, spec.kv_heads))
        self.spec, self.dtype, self.eps = spec, dtype, cfg.norm_eps

        def col(n, k=D):
            return ColumnParallelLinear(k, n, tp_size=tp, dtype=dtype)

        self.q_proj, self.k_proj = (col(spec.kv_heads * d) for _ in range(2))
        self.v_proj, self.b_proj = col(spec.heads * e), col(spec.heads)
        self.a1_proj = ops.Linear(D, spec.decay_rank, bias=False, dtype=dtype)
        self.g1_proj = ops.Linear(D, spec.gate_rank, bias=False, dtype=dtype)
        self.a2_proj = col(spec.heads * d, spec.decay_rank)
        self.g2_proj = col(spec.heads * e, spec.gate_rank)
        self.o_proj = RowParallelLinear(spec.heads * e, D, tp_size=tp,
                                        dtype=dtype)

        def conv(n):               # the current token passes
            w = torch.zeros(n, spec.conv, dtype=dtype)
            w[:, -1] = 1
            return nn.Parameter(w)

        self.q_conv, self.k_conv, self.v_conv = (
            conv(n) for n in (G * d, G * d, H * e))
        self.a_log = _vector(H, 0, dtype)
        self.dt_bias = _vector(H * d, -2, dtype)
        self.norm = ops.RMSNorm(e, eps=cfg.norm_eps, dtype=dtype)
        self.lay = DR.DeltaLayout(H, G, d, e, spec.conv, spec.decay_rank,
                                  spec.gate_rank)
        self.n_z = ops.pad_to(self.lay.n_o, 32)
        self.expandable = DR.delta_chunk_supported(self.lay, dtype)

    def fuse(self):
        lay = self.lay
        self.in_rows = DR.pack_in(lay, *(m.weight.data for m in (
            self.q_proj, self.k_proj, self.v_proj, self.b_proj,
            self.a1_proj, self.g1_proj)))
        self.second_w = DR.pack_second(lay, self.a2_proj.weight.data,
                                       self.g2_proj.weight.data)
        self.conv_w = DR.pack_conv(lay, self.q_conv.data, self.k_conv.data,
                                   self.v_conv.data)
        self.decay = DR.pack_decay(lay, self.a_log.data, self.dt_bias.data)
        self.norm_w = pad(self.norm.weight.data.float(),
                          (0, lay.vc - lay.vdim)).contiguous()
        o = QK.pack_columns(self.o_proj.weight.data, lay.heads, lay.vdim,
                            lay.vc)
        self.out_w = pad(o, (0, self.n_z - lay.n_o)).contiguous()
        return [self.second_w]

    def forward(self, y, batch, cache, rope):
        lay = self.lay
        y2 = ops.fast_linear(y[:, lay.off_r:lay.n_y].contiguous(),
                             self.second_w)
        o = torch.empty(y.shape[0], lay.n_o, dtype=torch.float32,
                        device=y.device)
        args = (y, y2, lay, self.conv_w, self.decay, cache, batch, o)
        if batch.n_short:
            DR.delta_step(*args)
        if batch.n_seqs > batch.n_short:
            DR.delta_chunk(*args)
        z, swz = _new_z(self, y, self.out_w, filled=True)
        DR.delta_out(o, lay, self.norm_w, y2, z, self.eps, swz, y, cache[1],
                     batch)
        return z

    def alloc_cache(self, num_blocks, num_slots, device):
        return DR.alloc_delta_state(num_slots, self.lay, device, self.dtype)

    def block_elements(self) -> int:
        return 0

    def state_bytes(self) -> int:
        lay = self.lay
        return 4 * lay.heads * lay.dc * lay.vc + \
            (lay.taps - 1) * lay.off_b * self.o_proj.weight.element_size()

    def covered(self) -> bool:
        return self.lay.dc <= DR.MAX_DIM and self.lay.vc <= DR.MAX_VALUE


class ChunkedAttention(nn.Module):
    """Parameters of the attention in a twin mixer."""

    def __init__(self, cfg: ModelConfig, spec: AttentionSpec, dtype, tp: int):
        super().__init__()
        D = cfg.hidden_size
        H, G = (_local(n, tp, "heads") for n in (spec.heads, spec.kv_heads))

        def col(n):
            return ColumnParallelLinear(D, n, tp_size=tp, dtype=dtype)

        self.q_proj = col(spec.heads * spec.dim)
        self.k_proj = col(spec.kv_heads * spec.dim)
        self.v_proj = col(spec.kv_heads * spec.vdim)
        self.o_proj = RowParallelLinear(spec.heads * spec.vdim, D, tp_size=tp,
                                        dtype=dtype)
        self.q_norm = ops.RMSNorm(spec.dim, eps=cfg.norm_eps, dtype=dtype)
        self.k_norm = ops.RMSNorm(spec.dim, eps=cfg.norm_eps, dtype=dtype)
        self.sink = _vector(H, 0, dtype)
        self.lay = QK.QKVLayout(H, G, spec.dim, spec.vdim, spec.rope_dims)


class MinGRU(nn.Module):
    """Parameters of the minGRU in a twin mixer."""

    def __init__(self, cfg: ModelConfig, spec: MinGRUSpec, dtype, tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.width = _local(spec.width, tp, "columns")

        def col(bias):
            return ColumnParallelLinear(D, spec.width, bias=bias, tp_size=tp,
                                        dtype=dtype)

        self.z_proj, self.x_proj, self.g_proj = col(True), col(True), col(False)
        self.o_proj = RowParallelLinear(spec.width, D, tp_size=tp,
                                        dtype=dtype)
        self.padded = ops.pad_to(self.width, 8)


class Twin(nn.Module):
    """Attention beside a minGRU (one mixer): their results stand side by
    side in z, so that one product brings both back and adds them."""

    def __init__(self, cfg: ModelConfig, spec: TwinSpec, dtype, tp: int):
        super().__init__()
        self.spec, self.dtype, self.eps = spec, dtype, cfg.norm_eps
        self.left = ChunkedAttention(cfg, spec.left, dtype, tp)
        self.right = MinGRU(cfg, spec.right, dtype, tp)
        self.lay = self.left.lay
        self.n_z = ops.pad_to(self.lay.n_z + self.right.padded, 32)
        self.expandable = SK.shared_kv_flash_supported(self.lay, dtype)

    def fuse(self):
        a, r, lay = self.left, self.right, self.lay
        n = r.padded - r.width
        self.in_rows = torch.cat(
            [QK.pack_qkv(lay, a.q_proj.weight.data, a.k_proj.weight.data,
                         a.v_proj.weight.data)] +
            [pad(m.weight.data, (0, 0, 0, n))
             for m in (r.z_proj, r.x_proj, r.g_proj)])
        left = QK.pack_columns(a.o_proj.weight.data, lay.heads, lay.vdim,
                               lay.vc)
        out = torch.cat([left, pad(r.o_proj.weight.data, (0, n))], dim=1)
        self.out_w = pad(out, (0, self.n_z - out.shape[1])).contiguous()
        self.norms = torch.stack([a.q_norm.weight.data,
                                  a.k_norm.weight.data]).float()
        self.sink = a.sink.data.float()
        self.bias = torch.stack([pad(m.bias.data.float(), (0, n))
                                 for m in (r.z_proj, r.x_proj)])
        return []

    def forward(self, y, batch, cache, rope):
        lay, spec, (kv, state) = self.lay, self.spec, cache
        z, swz = _new_z(self, y, self.out_w,
                        filled=self.n_z == lay.n_z + self.right.padded)
        QK.qkv_prep(y, lay, *rope, batch.positions, batch.slots, kv,
                    self.norms, self.eps)
        args = (y, lay, kv, batch, spec.left.scale, None, z)
        kw = dict(chunk=spec.left.chunk, sink=self.sink,
                  out_scale=spec.left_scale)
        if batch.n_short:
            SK.shared_kv_attend(*args, swz, **kw)
        if batch.n_seqs > batch.n_short:
            SK.shared_kv_flash(*args, **kw)
        MG.min_gru(y, lay.n_y, self.bias, state, batch, z, lay.n_z,
                   spec.right_scale, swz)
        return z

    def alloc_cache(self, num_blocks, num_slots, device):
        return (SK.alloc_shared_kv_cache(num_blocks, self.lay, device,
                                         self.dtype),
                torch.zeros(num_slots, self.right.padded, device=device))

    def block_elements(self) -> int:
        return self.lay.kv_heads * self.lay.ec * ops.BLOCK_SIZE

    def state_bytes(self) -> int:
        return 4 * self.right.padded

    def covered(self) -> bool:
        return max(self.lay.hc, self.lay.vc) <= SK.MAX_HEAD


class SquaredRelu(nn.Module):
    """down(relu(up)^2)."""

    def __init__(self, cfg: ModelConfig, ff: int, dtype, tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.ff = _local(ff, tp, "columns")
        self.fc = ops.pad_to(self.ff, 32)
        self.up_proj = ColumnParallelLinear(D, ff, tp_size=tp, dtype=dtype)
        self.down_proj = RowParallelLinear(ff, D, tp_size=tp, dtype=dtype)

    def fuse(self):
        n = self.fc - self.ff
        self.in_rows = pad(self.up_proj.weight.data, (0, 0, 0, n))
        self.out_w = pad(self.down_proj.weight.data, (0, n)).contiguous()
        return []

    def forward(self, h, y):
        """(result, further parts of it)"""
        z = ops.squared_relu(y, self.fc,
                             ops.decode_ready(self.out_w, y.shape[0]))
        return _project(z, self.out_w, 1), None


class Mixture(nn.Module):
    """Experts and, optionally, a shared unit."""

    def __init__(self, cfg: ModelConfig, spec: MoESpec, dtype, tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.spec = spec
        self.router = ops.Linear(D, spec.experts, bias=False, dtype=dtype)
        self.correction = _vector(spec.experts, 0, dtype)
        self.experts = nn.ModuleList(SquaredRelu(cfg, spec.ff, dtype, tp)
                                     for _ in range(spec.experts))
        self.shared = (SquaredRelu(cfg, spec.shared_ff, dtype, tp)
                       if spec.shared_ff else None)

    @torch.no_grad()
    def fuse(self):
        k = -self.router.weight.shape[1] % 32
        e0, E = self.experts[0], self.spec.experts
        self.router_w = pad(self.router.weight.data,
                            (0, k, 0, -E % 32)).contiguous()
        self.choice = self.correction.data.float()
        D = self.router.weight.shape[1]
        up = e0.up_proj.weight.new_zeros(E, e0.fc, D + k)
        down = up.new_zeros(E, D, e0.fc)
        for i, e in enumerate(self.experts):
            u, d = up[i, :e.ff, :D], down[i, :, :e.ff]
            u.copy_(e.up_proj.weight)
            d.copy_(e.down_proj.weight)
            e.up_proj.weight = nn.Parameter(u, requires_grad=False)
            e.down_proj.weight = nn.Parameter(d, requires_grad=False)
        self.up_w, self.down_w = up, down
        self.in_rows = up.new_zeros(0, D)
        more = []
        if self.shared is not None:
            more = self.shared.fuse()
            self.in_rows = self.shared.in_rows
        return [self.router_w, *more] + \
            ([self.shared.out_w] if self.shared is not None else [])

    def forward(self, h, y):
        s = self.spec
        logits = _project(h, self.router_w, 1)
        plan = ME.moe_plan(
            ME.moe_route(logits, self.choice, s.top, s.groups, s.keep),
            s.experts, h.dtype == torch.bfloat16)
        parts = ME.moe_down(ME.moe_up(h, self.up_w, plan), self.down_w, plan)
        return parts, (None if self.shared is None
                       else self.shared(h, y)[0])


class Join(nn.Module):
    """How a sublayer reads the streams and how its result comes back."""

    def __init__(self, cfg: ModelConfig, dtype):
        super().__init__()
        D, s = cfg.hidden_size, cfg.streams
        self.scale = _vector(D, 1, dtype)
        self.gate = ops.Linear(D, D, bias=True, dtype=dtype)
        self.inp, self.out = _vector(s, 1 / s, dtype), _vector(s, 1, dtype)
        self.mix = nn.Parameter(torch.eye(s, dtype=dtype))
        self.mult = cfg.residual_mult

    def fuse(self):
        self.inp_v = self.inp.data.float()
        self.packed = ST.pack_join(self.scale.data, self.gate.bias.data,
                                   self.out.data, self.mix.data, self.mult)


class StreamBlock(nn.Module):
    def __init__(self, cfg: ModelConfig, spec: LayerSpec, dtype, tp: int):
        super().__init__()
        self.spec, self.tp, self.dtype = spec, tp, dtype
        self.norm1 = ops.DynamicTanh(cfg.hidden_size, dtype=dtype)
        self.join1 = Join(cfg, dtype)
        mixer = GatedDelta if isinstance(spec.mixer, GatedDeltaSpec) else Twin
        self.mixer = mixer(cfg, spec.mixer, dtype, tp)
        self.parts = [(self.norm1, self.join1, self.mixer)]
        if spec.mlp is not None:
            self.norm2 = ops.DynamicTanh(cfg.hidden_size, dtype=dtype)
            self.join2 = Join(cfg, dtype)
            self.mlp = (SquaredRelu(cfg, spec.mlp.ff, dtype, tp)
                        if isinstance(spec.mlp, SquaredReluSpec)
                        else Mixture(cfg, spec.mlp, dtype, tp))
            self.parts.append((self.norm2, self.join2, self.mlp))

    @property
    def expandable(self) -> bool:
        return self.mixer.expandable

    @torch.no_grad()
    def fuse(self) -> list[torch.Tensor]:
        """Serving weights from the loaded parameters; returns those the
        decode GEMM may keep a copy of."""
        weights = []
        for norm, join, part in self.parts:
            weights += part.fuse()
            join.fuse()
            join.norm_v = norm.packed()
            D = join.scale.numel()
            rows = torch.cat([part.in_rows, join.gate.weight.data])
            join.off = part.in_rows.shape[0]
            del part.in_rows
            join.in_w = pad(rows, (0, -D % 32, 0, -rows.shape[0] % 32)
                            ).contiguous()
            # the gate's rows stand in the joint weight as they are
            join.gate.weight = nn.Parameter(
                join.in_w[join.off:join.off + D, :D], requires_grad=False)
            weights.append(join.in_w)
            if hasattr(part, "out_w"):
                weights.append(part.out_w)
        return weights

    def step(self, x, pending, batch, cache, rope, contexts):
        """x [T, streams, D] fp32 before `pending`, the last sublayer's
        result; adds it to x in place and returns this layer's own."""
        T = x.shape[0]
        for _, join, part in self.parts:
            h = ops.streams_norm(x, pending, join.inp_v, join.norm_v,
                                 self.dtype,
                                 operand=ops.decode_ready(join.in_w, T))
            y = ops.fast_linear(h, join.in_w)
            if part is self.mixer:
                z = part(y, batch, cache, rope)
                delta, extra = _project(z, part.out_w, self.tp), None
            else:
                delta, extra = part(h, y)
                if self.tp > 1:
                    parts = [d if d.dim() == 3 else d[None]
                             for d in (delta, extra) if d is not None]
                    delta = reduce_from_tp(torch.cat(parts).sum(0))
                    extra = None
            pending = ops.Pending(delta, extra, y, join.off, join.packed)
        return pending

    def alloc_cache(self, num_blocks: int, num_slots: int, device):
        return self.mixer.alloc_cache(num_blocks, num_slots, device)

    def block_elements(self) -> int:
        return self.mixer.block_elements()

    def state_bytes(self) -> int:
        return self.mixer.state_bytes()

    def covered(self) -> bool:
        """The kernels run these sizes."""
        s, mlp = self.join1.inp.numel(), self.spec.mlp
        return self.mixer.covered() and s <= ST.MAX_STREAMS and not (
            isinstance(mlp, MoESpec) and
            (mlp.experts > ME.MAX_EXPERTS or mlp.top > ME.MAX_TOP))
