"""SiluAndMul with the reference's interface (nanovllm/layers/activation.py:6-16), computed by the
HIP kernel ``nv_silu_and_mul``: one launch instead of the silu and multiply kernels."""
from __future__ import annotations

import torch
from torch import nn

from .. import ops


class SiluAndMul(nn.Module):
    def __init__(self):
        super().__init__()

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.silu_and_mul(x)


class GeluTanhAndMul(nn.Module):
    """gelu_tanh(gate) * up for x = [gate | up] (the HIP kernel ``nv_gelu_tanh_and_mul``; bfloat16 or float32)."""

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.gelu_tanh_and_mul(x)


class SiluAndMulRows(nn.Module):
    """silu(gate) * up for x = [gate | up] of any width (the HIP kernel ``nv_silu_and_mul_rows``; bfloat16 or float32)."""

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.silu_and_mul_rows(x)


class ClampedGLU(nn.Module):
    """g sigmoid(alpha g) (u + shift) with g = min(gate, limit), u = clamp(up, -limit, limit) for x = [gate | up] of any width
    (the HIP kernel ``nv_clamped_glu_rows``; bfloat16 or float32)."""

    def __init__(self, limit: float, alpha: float = 1.702, shift: float = 1.0):
        super().__init__()
        self.limit, self.alpha, self.shift = float(limit), float(alpha), float(shift)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.clamped_glu_rows(x, self.limit, self.alpha, self.shift)


class ScaledSoftcap(nn.Module):
    """cap * tanh(scale * x / cap) in float32; cap 0: scale * x (the HIP kernel ``nv_scale_softcap``)."""

    def __init__(self, scale: float, cap: float):
        super().__init__()
        self.scale, self.cap = float(scale), float(cap)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return ops.scale_softcap(x, self.scale, self.cap)
