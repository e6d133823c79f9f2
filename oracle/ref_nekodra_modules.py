"""Oracle (test infrastructure): torch stand-ins for the layers Nekodra is built from (token + position embedding, the
two-layer-norm stream boundary with routed parts, layer norm, latent attention without positions over the paged latent
cache, per-head products, softmax routing with identity experts, SiLU experts), with the same constructors and the same
cache layouts as the HIP-backed modules.  They let the whole engine run without a GPU and give GPU tests an eager
reference per layer.  Device-agnostic, slow, written from the layer interfaces; the product model never imports it."""
from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

from .ref_benarax_modules import _ctx, _unit_rms
from .ref_divadra_modules import _spans


class PositionEmbedding(nn.Module):
    def __init__(self, vocab, max_positions, width, dtype=None, device=None):
        super().__init__()
        self.weight = nn.Parameter(torch.zeros(vocab, width, dtype=dtype, device=device))
        self.pos = nn.Parameter(torch.zeros(max_positions, width, dtype=dtype, device=device))

    def forward(self, ids, positions):
        return self.weight[ids].float() + self.pos[positions].float()


class LayerNorm(nn.Module):
    def __init__(self, width, eps=1e-5, device=None):
        super().__init__()
        self.eps = eps
        self.weight = nn.Parameter(torch.ones(width, dtype=torch.float32, device=device))
        self.bias = nn.Parameter(torch.zeros(width, dtype=torch.float32, device=device))


def layernorm_pair_boundary(x, adds=(), routed=None, norm_a=None, norm_b=None, eps=1e-5, out_dtype=None, want_f32_b=False):
    for a in adds:
        x += a.float()
    if routed is not None:
        parts, ids, weights, experts, through = routed
        for j in range(parts.shape[1]):
            if ids is None:
                x += parts[:, j]
                continue
            product = (ids[:, j] < experts)[:, None]
            other = through.float() * weights[:, j][:, None] if through is not None else torch.zeros_like(x)
            x += torch.where(product, parts[:, j], other)
    d = x - x.mean(-1, keepdim=True)
    u = d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps)
    a = (u * norm_a[0] + norm_a[1]).to(out_dtype or torch.float32) if norm_a is not None else None
    b32 = u * norm_b[0] + norm_b[1] if norm_b is not None else None
    b = b32.to(out_dtype or torch.float32) if b32 is not None else None
    return a, b, (b32 if want_f32_b else None)


class SiluAndMulRows(nn.Module):
    def forward(self, x):
        g, u = x.float().chunk(2, dim=-1)
        return (g * torch.sigmoid(g) * u).to(x.dtype)


class UnrotatedLatentAttention(nn.Module):
    def __init__(self, num_heads, rank, scale, eps, own_latent=True, use_sink=False, device=None):
        super().__init__()
        self.H, self.rank, self.scale, self.eps = num_heads, rank, float(scale), eps
        f32 = dict(dtype=torch.float32, device=device)
        self.latent_norm = nn.Parameter(torch.ones(rank, **f32)) if own_latent else None
        self.sink = nn.Parameter(torch.zeros(num_heads, **f32)) if use_sink else None

    def forward(self, q_lat, c_raw, k_cache, v_cache):
        ctx = _ctx()
        dt, T, H, rank = q_lat.dtype, q_lat.shape[0], self.H, self.rank
        if self.latent_norm is not None:
            c = (_unit_rms(c_raw.float(), self.eps) * self.latent_norm).to(dt)
            k_cache.view(-1, rank)[ctx.slot_mapping.long()] = c
        bs = k_cache.shape[1]
        q = q_lat.view(T, H, rank).float()
        out = torch.zeros(T, H, rank, dtype=torch.float32, device=q.device)
        for b, _, r0, nq, start in _spans(ctx):
            pos_k = torch.arange(start + nq, device=q.device)
            rows = ctx.block_tables[b].long()[pos_k // bs] * bs + pos_k % bs
            c = k_cache.view(-1, rank)[rows].float()
            pos_q = start + torch.arange(nq, device=q.device)
            for h in range(H):
                s = (q[r0:r0 + nq, h] @ c.t() * self.scale).masked_fill(pos_q[:, None] < pos_k[None, :], float("-inf"))
                if self.sink is not None:
                    s = torch.cat([s, self.sink[h].expand(nq, 1)], dim=1)
                out[r0:r0 + nq, h] = torch.softmax(s, dim=-1)[:, :start + nq] @ c
        return out.reshape(T, H * rank).to(dt)


class HeadLinear(nn.Module):
    def __init__(self, heads, n_in, n_out, dtype=None, device=None):
        super().__init__()
        self.weight = nn.Parameter(torch.zeros(heads, n_out, n_in, dtype=dtype, device=device))

    def forward(self, x, gate=None):
        H, N, K = self.weight.shape
        x = x.reshape(-1, H, K).float()
        y = torch.cat([x[:, h] @ self.weight[h].float().t() for h in range(H)], dim=1)
        if gate is not None:
            y = y * torch.sigmoid(gate.float())
        return y.to(self.weight.dtype)


class SoftmaxRouter(nn.Module):
    def __init__(self, experts, top, scale=1.0, device=None):
        super().__init__()
        self.experts, self.top, self.scale = int(experts), int(top), float(scale)
        self.correction = nn.Parameter(torch.zeros(experts, dtype=torch.float32, device=device))

    def forward(self, logits):
        s = torch.softmax(logits.float(), dim=-1)
        ids = (s + self.correction if self.correction is not None else s).topk(self.top, dim=-1).indices
        return ids.to(torch.int32), s.gather(1, ids) * self.scale


class SiluExperts(nn.Module):
    def forward(self, h, ids, weights, gate_up, down):
        T, top, dt, ff = h.shape[0], ids.shape[1], h.dtype, gate_up.shape[1] // 2
        out = torch.full((T, top, down.shape[1]), float("nan"), dtype=torch.float32, device=h.device)   # unwritten rows
        for e in range(gate_up.shape[0]):
            t, j = (ids == e).nonzero(as_tuple=True)
            if t.numel() == 0:
                continue
            gu = F.linear(h[t], gate_up[e]).float()
            y = (gu[:, :ff] * torch.sigmoid(gu[:, :ff]) * gu[:, ff:]).to(dt)
            out[t, j] = F.linear(y, down[e]).float() * weights[t, j][:, None]
        return out
