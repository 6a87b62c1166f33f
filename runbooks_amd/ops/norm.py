"""RMSNorm and LayerNorm: fused gfx950 HIP kernels (GPU) / fp32 references
(CPU)."""
from __future__ import annotations

import torch

from . import _backend


def rmsnorm_ref(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """Plain PyTorch fp32 reference (llama-family RMSNorm semantics)."""
    xf = x.float()
    var = xf.pow(2).mean(-1, keepdim=True)
    y = xf * torch.rsqrt(var + eps)
    return (y * weight.float()).to(x.dtype)


class _RMSNormFn(torch.autograd.Function):
    @staticmethod
    def forward(ctx, x, weight, eps):
        y, inv_rms = _backend.ext().rmsnorm_fwd(x, weight, eps)
        ctx.save_for_backward(x, weight, inv_rms)
        return y

    @staticmethod
    def backward(ctx, dy):
        x, weight, inv_rms = ctx.saved_tensors
        dx, dw = _backend.ext().rmsnorm_bwd(x, weight, dy.contiguous(), inv_rms)
        return dx, dw.to(weight.dtype), None


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    if _backend.use_hip(x):
        if (not torch.is_grad_enabled() and x.dtype == torch.bfloat16
                and x.numel() // x.shape[-1] <= 32
                and x.shape[-1] % 16 == 0):
            # decode-shaped rows: one pass also emits the decode GEMM's
            # pre-swizzled operand (csrc/decode_gemm.hip), saving the
            # standalone x-swizzle launch on the consumer side
            y, swz = _backend.ext().rmsnorm_fwd_dec(
                x.contiguous(), weight.contiguous(), eps)
            y._rb_swz = swz
            return y
        return _RMSNormFn.apply(x.contiguous(), weight.contiguous(), eps)
    return rmsnorm_ref(x, weight, eps)


def rmsnorm_res32(x: torch.Tensor, delta: torch.Tensor | None,
                  weight: torch.Tensor, eps: float, dtype: torch.dtype,
                  operand: bool = False, offset: float = 0.0
                  ) -> torch.Tensor:
    """Norm of a 32-bit residual: x [T, D] fp32 += delta in place, returns
    rmsnorm(x) * (offset + weight) in `dtype`. delta: fp32 or `dtype` [T, D], an
    uncombined fp32 split-K slab [split, T, D], or None. operand=True also
    attaches the decode GEMM's pre-swizzled operand (T <= 32)."""
    if not _backend.use_hip(x):
        if delta is not None:
            x += delta.float() if delta.dim() == 2 else delta.sum(0)
        return rmsnorm_ref(x, offset + weight.float(), eps).to(dtype)
    y, swz = _backend.ext().rmsnorm_res32(
        x, None if delta is None else delta.contiguous(), weight, eps,
        operand, offset)
    if operand:
        y._rb_swz = swz
    return y


def layernorm_ref(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor,
                  eps: float) -> torch.Tensor:
    d = x.float()
    d = d - d.mean(-1, keepdim=True)
    y = d * torch.rsqrt(d.pow(2).mean(-1, keepdim=True) + eps)
    return (y * weight.float() + bias.float()).to(x.dtype)


def layernorm_res32(x: torch.Tensor, delta: torch.Tensor | None,
                    weight: torch.Tensor, bias: torch.Tensor, eps: float,
                    dtype: torch.dtype, operand: bool = False
                    ) -> torch.Tensor:
    """rmsnorm_res32 with a layer norm (mean taken off, bias added)."""
    if not _backend.use_hip(x):
        if delta is not None:
            x += delta.float() if delta.dim() == 2 else delta.sum(0)
        return layernorm_ref(x, weight, bias, eps).to(dtype)
    y, swz = _backend.ext().layernorm_res32(
        x, None if delta is None else delta.contiguous(), weight, bias, eps,
        operand)
    if operand:
        y._rb_swz = swz
    return y


def norm_res32(norm: torch.nn.Module, x: torch.Tensor,
               delta: torch.Tensor | None, dtype: torch.dtype,
               operand: bool = False) -> torch.Tensor:
    """x += delta, then `norm` (an RMSNorm, or a LayerNorm with bias)."""
    bias = getattr(norm, "bias", None)
    if bias is None:
        return rmsnorm_res32(x, delta, norm.weight, norm.eps, dtype, operand,
                             norm.offset)
    return layernorm_res32(x, delta, norm.weight, bias, norm.eps, dtype,
                           operand)


def join_res32(x: torch.Tensor, delta: torch.Tensor | None,
               other: torch.Tensor, operand: bool = False) -> torch.Tensor:
    """[x + delta ; other] in other's dtype, [T, 2 D] (x fp32 is left as it
    is): the input of a projection that replaces the residual. operand=True
    also attaches the decode GEMM's operand."""
    if not _backend.use_hip(x):
        if delta is not None:
            x = x + (delta.float() if delta.dim() == 2 else delta.sum(0))
        return torch.cat([x.to(other.dtype), other], dim=-1)
    y, swz = _backend.ext().join_res32(
        x, None if delta is None else delta.contiguous(), other, operand)
    if operand:
        y._rb_swz = swz
    return y


class RMSNorm(torch.nn.Module):
    """`offset` is added to the stored weight (served residual norms
    only)."""

    def __init__(self, dim: int, eps: float = 1e-5, dtype=None,
                 offset: float = 0.0):
        super().__init__()
        self.weight = torch.nn.Parameter(
            torch.full((dim,), 1.0 - offset, dtype=dtype))
        self.eps, self.offset = eps, offset

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        if self.offset:
            raise NotImplementedError("RMSNorm.forward with an offset")
        return rmsnorm(x, self.weight, self.eps)

    def extra_repr(self) -> str:
        return f"dim={self.weight.numel()}, eps={self.eps}"
