"""Layers of models described layer by layer whose sublayers follow each
other: windowed attention on shared keys and values, or lightning attention,
then (optionally) a gated MLP, each behind a norm of its own and added to a
32-bit residual.

A sublayer runs as two products around its mechanism (ops/shared_kv.py,
ops/lightning.py, the gated unit); the second one's fp32 result, or the
decode GEMM's uncombined split-K slab, is added by the norm that follows.
`fuse()` builds the serving weights from the loaded parameters.

Tensor parallelism: heads and MLP columns are sharded, one all-reduce per
sublayer; the lightning norm over all heads adds one of a float per token.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import ops
from ..ops import lightning as LA
from ..ops import shared_kv as SK
from ..parallel import (ColumnParallelLinear, RowParallelLinear, comm,
                        reduce_from_tp)
from .config import (GLUSpec, LayerSpec, LightningSpec, ModelConfig,
                     SharedKVAttentionSpec)


def _project(z, w, tp: int):
    """The sublayer's pending output: fp32, or a split-K slab."""
    if tp == 1 and ops.decode_ready(w, z.shape[0]):
        return ops.decode_linear_raw(z, w, f32=True)[0]
    out = ops.linear_f32_parts(z, w)
    if tp == 1:
        return out
    return reduce_from_tp(out if out.dim() == 2 else out.sum(0))


def _new_z(lay, y, w, filled: bool):
    """z and, where its product runs on the decode GEMM, that operand;
    zeroed unless the kernel fills every column."""
    T = y.shape[0]
    make = torch.empty if filled else torch.zeros
    z = make(T, lay.n_z, dtype=y.dtype, device=y.device)
    if not ops.decode_ready(w, T):
        return z, None
    swz = ops.decode_operand(T, lay.n_z, z)
    if not filled:
        swz.zero_()
    z._rb_swz = swz
    return z, swz


class SharedKVAttention(nn.Module):
    """Attention on shared keys and values (one mixer)."""

    def __init__(self, cfg: ModelConfig, spec: SharedKVAttentionSpec, dtype,
                 tp: int):
        super().__init__()
        if spec.heads % tp or spec.kv_heads % tp:
            raise ValueError(f"{spec.heads} / {spec.kv_heads} heads do not "
                             f"divide tp={tp}")
        D, d = cfg.hidden_size, spec.dim
        self.spec, self.dtype = spec, dtype
        self.q_proj = ColumnParallelLinear(D, spec.heads * d, tp_size=tp,
                                           dtype=dtype)
        self.k_proj = ColumnParallelLinear(D, spec.kv_heads * d, tp_size=tp,
                                           dtype=dtype)
        self.o_proj = RowParallelLinear(spec.heads * d, D, tp_size=tp,
                                        dtype=dtype)
        self.lay = SK.SharedKVLayout(spec.heads // tp, spec.kv_heads // tp, d,
                                     spec.rope_dims)
        self.expandable = SK.shared_kv_flash_supported(self.lay, dtype)

    def fuse(self):
        self.in_w = SK.pack_in(self.lay, self.q_proj.weight.data,
                               self.k_proj.weight.data)
        self.out_w = SK.pack_out(self.lay, self.o_proj.weight.data)

    def forward(self, h, batch, cache, rope):
        lay, spec = self.lay, self.spec
        y = ops.fast_linear(h, self.in_w)
        z, swz = _new_z(lay, y, self.out_w,
                        filled=lay.n_z == lay.heads * lay.hc)
        SK.shared_kv_prep(y, lay, *rope, batch.positions, batch.slots, cache)
        if batch.n_short:
            SK.shared_kv_attend(y, lay, cache, batch, spec.scale, spec.window,
                                z, swz)
        if batch.n_seqs > batch.n_short:
            SK.shared_kv_flash(y, lay, cache, batch, spec.scale, spec.window,
                               z)
        return z

    def alloc_cache(self, num_blocks, num_slots, device):
        return SK.alloc_shared_kv_cache(num_blocks, self.lay, device,
                                        self.dtype)

    def block_elements(self) -> int:
        return self.lay.kv_heads * self.lay.ec * ops.BLOCK_SIZE

    def covered(self) -> bool:
        return self.lay.hc <= SK.MAX_HEAD


class LightningAttention(nn.Module):
    """Linear attention with a decayed state (one mixer)."""

    def __init__(self, cfg: ModelConfig, spec: LightningSpec, dtype, tp: int):
        super().__init__()
        if spec.heads % tp:
            raise ValueError(f"{spec.heads} heads do not divide tp={tp}")
        D, H = cfg.hidden_size, spec.heads
        self.spec, self.dtype, self.tp, self.eps = spec, dtype, tp, cfg.norm_eps

        def col(n):
            return ColumnParallelLinear(D, n, tp_size=tp, dtype=dtype)

        self.q_proj, self.k_proj = col(H * spec.dim), col(H * spec.dim)
        self.v_proj, self.g_proj = col(H * spec.vdim), col(H * spec.vdim)
        self.o_proj = RowParallelLinear(H * spec.vdim, D, tp_size=tp,
                                        dtype=dtype)
        h = H // tp
        self.norm = ops.RMSNorm(h * spec.vdim, eps=cfg.norm_eps, dtype=dtype)
        self.lay = LA.LightningLayout(h, spec.dim, spec.vdim)
        first = comm.rank() * h if tp > 1 else 0
        self.register_buffer("powers", LA.decay_powers(
            spec.decay[first:first + h], torch.get_default_device()),
            persistent=False)
        self.expandable = LA.lightning_chunk_supported(self.lay, dtype)

    def fuse(self):
        self.in_w = LA.pack_in(self.lay, self.q_proj.weight.data,
                               self.k_proj.weight.data,
                               self.v_proj.weight.data,
                               self.g_proj.weight.data)
        self.norm_w = LA.pack_norm(self.lay, self.norm.weight.data)
        self.out_w = LA.pack_out(self.lay, self.o_proj.weight.data)

    def forward(self, h, batch, state, rope):
        lay = self.lay
        y = ops.fast_linear(h, self.in_w)
        o = torch.empty(y.shape[0], lay.n_o, dtype=torch.float32,
                        device=y.device)
        if batch.n_short:
            LA.lightning_step(y, lay, state, batch, self.powers, o)
        if batch.n_seqs > batch.n_short:
            LA.lightning_chunk(y, lay, state, batch, self.powers, o)
        sums = None
        if self.tp > 1:
            sums = reduce_from_tp(o.pow(2).sum(-1))
        z, swz = _new_z(lay, y, self.out_w, filled=True)
        LA.lightning_out(o, lay, self.norm_w, y, z,
                         self.spec.heads * self.spec.vdim, self.eps, sums, swz)
        return z

    def alloc_cache(self, num_blocks, num_slots, device):
        return ops.alloc_lightning_state(num_slots, self.lay, device)

    def block_elements(self) -> int:
        return 0

    def covered(self) -> bool:
        return self.lay.dc <= LA.MAX_DIM


class GatedGelu(nn.Module):
    """Gated unit with a tanh-GELU."""

    def __init__(self, cfg: ModelConfig, spec: GLUSpec, dtype, tp: int):
        super().__init__()
        D = cfg.hidden_size
        self.ff = spec.ff // tp
        self.fc = ops.pad_to(self.ff, 16)
        self.gate_proj = ColumnParallelLinear(D, spec.ff, tp_size=tp,
                                              dtype=dtype)
        self.up_proj = ColumnParallelLinear(D, spec.ff, tp_size=tp,
                                            dtype=dtype)
        self.down_proj = RowParallelLinear(spec.ff, D, tp_size=tp,
                                           dtype=dtype)

    def fuse(self):
        pad = nn.functional.pad
        n = self.fc - self.ff
        self.in_w = torch.cat([pad(m.weight.data, (0, 0, 0, n)) for m in
                               (self.gate_proj, self.up_proj)]).contiguous()
        self.out_w = pad(self.down_proj.weight.data, (0, n)).contiguous()

    def forward(self, h):
        return ops.geglu(ops.fast_linear(h, self.in_w),
                         operand=ops.decode_ready(self.out_w, h.shape[0]))


class SequentialBlock(nn.Module):
    def __init__(self, cfg: ModelConfig, spec: LayerSpec, dtype, tp: int):
        super().__init__()
        self.spec, self.tp, self.dtype = spec, tp, dtype

        def norm():
            if cfg.norm == "layernorm":
                return nn.LayerNorm(cfg.hidden_size, eps=cfg.norm_eps,
                                    dtype=dtype)
            return ops.RMSNorm(cfg.hidden_size, eps=cfg.norm_eps, dtype=dtype)

        self.norm1 = norm()
        mixer = (LightningAttention if isinstance(spec.mixer, LightningSpec)
                 else SharedKVAttention)
        self.mixer = mixer(cfg, spec.mixer, dtype, tp)
        if spec.mlp is not None:
            self.norm2 = norm()
            self.mlp = GatedGelu(cfg, spec.mlp, dtype, tp)

    @property
    def expandable(self) -> bool:
        return self.mixer.expandable

    @torch.no_grad()
    def fuse(self) -> list[torch.Tensor]:
        """Serving weights from the loaded parameters; returns those the
        decode GEMM may keep a copy of."""
        parts = [self.mixer] + ([self.mlp] if self.spec.mlp else [])
        for p in parts:
            p.fuse()
            own = [m for m in p.children()
                   if isinstance(m, ColumnParallelLinear)]
            self._adopt(p.in_w, own)
            if p.out_w.shape == self._out(p).weight.shape and \
                    torch.equal(p.out_w, self._out(p).weight):
                self._out(p).weight = nn.Parameter(p.out_w,
                                                   requires_grad=False)
        return [w for p in parts for w in (p.in_w, p.out_w)]

    @staticmethod
    def _out(part):
        return part.o_proj if hasattr(part, "o_proj") else part.down_proj

    @staticmethod
    def _adopt(wide, linears):
        """Parameters whose rows the joint weight holds unpadded become
        views of it."""
        if wide.shape[0] != sum(m.weight.shape[0] for m in linears):
            return
        at = 0
        for m in linears:
            n = m.weight.shape[0]
            m.weight = nn.Parameter(wide[at:at + n], requires_grad=False)
            at += n

    def step(self, x, delta, batch, cache, rope, contexts):
        """x [T, D] fp32 residual before this layer without `delta`, the
        last sublayer's pending output; adds delta to x in place and returns
        this layer's own pending output."""
        T = x.shape[0]

        def normed(norm, w):
            return ops.norm_res32(norm, x, delta, self.dtype,
                                  operand=ops.decode_ready(w, T))

        h = normed(self.norm1, self.mixer.in_w)
        delta = _project(self.mixer(h, batch, cache, rope), self.mixer.out_w,
                         self.tp)
        if self.spec.mlp is None:
            return delta
        h = normed(self.norm2, self.mlp.in_w)
        return _project(self.mlp(h), self.mlp.out_w, self.tp)

    def alloc_cache(self, num_blocks: int, num_slots: int, device):
        return self.mixer.alloc_cache(num_blocks, num_slots, device)

    def block_elements(self) -> int:
        """Cached elements of one block of tokens."""
        return self.mixer.block_elements()

    def covered(self) -> bool:
        """The kernels run heads of this size."""
        return self.mixer.covered()

    def state_bytes(self) -> int:
        """Bytes a sequence's state takes."""
        lay = self.mixer.lay
        return (0 if self.spec.attends
                else 4 * lay.heads * lay.dc * lay.vc)
