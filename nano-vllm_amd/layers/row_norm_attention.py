"""Causal softmax attention over the paged KV cache whose queries and keys are RMS-normed over the WHOLE projection, and the
step that hands two mixers' outputs to one output product, backed by gfx950 HIP kernels.

``RowNormAttention``: q and k are divided by the root mean square of their whole row (all heads at once), times one weight
per column, then rotated on the first rot_dims dimensions of every head (rotate-half pairs; the frequencies may be blended
for long contexts, which also gives cos and sin a magnitude); free key and value sizes; scores scale * q . k in float32,
ordinary softmax over the visible keys (the score-modified kernel family with every modifier off).  ``JoinGated``: the heads
of an attention times one sigmoid gate each, a linear memory's read-out RMS-normed over its row times a weight and a sigmoid
gate per column, each side times a constant, side by side as the rows of one product.
"""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from ..utils.cache_context import get_context
from .latent_attention import blended_frequencies


class RowNormAttention(nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, head_dim: int, v_head_dim: int, scale: float, eps: float,
                 rot_dims: int = 0, rot_base: float = 10000.0, rot_scaling: dict | None = None, device=None):
        super().__init__()
        assert num_heads % num_kv_heads == 0 and rot_dims % 2 == 0 and rot_dims <= head_dim
        self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim = num_heads, num_kv_heads, head_dim, v_head_dim
        self.scale, self.eps, self.rot_dims = float(scale), float(eps), int(rot_dims)
        f32 = dict(dtype=torch.float32, device=device)
        self.q_norm = nn.Parameter(torch.ones(num_heads * head_dim, **f32))
        self.k_norm = nn.Parameter(torch.ones(num_kv_heads * head_dim, **f32))
        freq, self.mag = blended_frequencies(rot_dims, rot_base, rot_scaling) if rot_dims else (None, 1.0)
        self.register_buffer("freq", freq.to(device) if freq is not None else None, persistent=False)

    def forward(self, q, k, v, positions, k_cache, v_cache) -> torch.Tensor:
        """q: [T, H, D]; k: [T, G, D]; v: [T, G, Dv] as projected; caches [num_blocks, block_size, G, D | Dv].  Returns
        [T, H * Dv]."""
        ctx = get_context()
        qp = ops.row_norm_rope_store(positions, q, k, v, self.q_norm, self.k_norm, self.eps, self.freq, self.rot_dims, self.mag,
                                     ctx.slot_mapping, k_cache, v_cache)
        singles = -1 if ctx.num_decode_seqs is None else int(ctx.num_decode_seqs > 0)
        return ops.attn_scoremod_paged(qp, k_cache, v_cache, ctx.cu_seqlens_q, ctx.cu_seqlens_k, ctx.block_tables,
                                       self.scale, 0.0, None, None, ctx.max_seqlen_q, ctx.max_seqlen_k, singles)


class JoinGated(nn.Module):
    def __init__(self, mem_cols: int, eps: float, left_scale: float, right_scale: float, device=None):
        super().__init__()
        self.eps, self.left_scale, self.right_scale = float(eps), float(left_scale), float(right_scale)
        self.norm_weight = nn.Parameter(torch.ones(mem_cols, dtype=torch.float32, device=device))

    def forward(self, attn, head_gate, mem, gate) -> torch.Tensor:
        """attn [T, H * Dv], head_gate [T, H] raw, mem [T, cols] float32, gate [T, cols] raw; returns [T, H * Dv + cols]."""
        return ops.join_gated(attn, head_gate, self.left_scale, mem, self.norm_weight, gate, self.eps, self.right_scale)
