"""Oracle (test infrastructure): torch stand-ins for the layers Tiralix is built from (the stream boundary with normed inputs,
scaled norm weights, the selective scan, attention with whole-row q / k norms, the fixed-decay memory, the gated join of two
mixers, the clamped gated unit, soft-capped logits), with the same constructors and the same cache / state layouts as the
HIP-backed modules.  They let the whole engine run without a GPU and give GPU tests an eager reference per layer.
Device-agnostic, slow, written from the layer interfaces; the product model never imports it."""
from __future__ import annotations

import math

import torch
import torch.nn as nn
import torch.nn.functional as F

from .ref_benarax_modules import _ctx, _unit_rms, stream_boundary  # noqa: F401
from .ref_divadra_modules import ConvBiasSilu, _spans, _turn  # noqa: F401


class ScaledNorm(nn.Module):
    def __init__(self, width, device=None):
        super().__init__()
        self.weight = nn.Parameter(torch.ones(width, dtype=torch.float32, device=device))
        self.scale = nn.Parameter(torch.ones(width, dtype=torch.float32, device=device))
        self.register_buffer("applied", torch.ones(width, dtype=torch.float32, device=device), persistent=False)

    def finalize(self):
        self.applied = self.weight.data * self.scale.data


class SelectiveScan(nn.Module):
    def __init__(self, channels, states, device=None):
        super().__init__()
        self.C, self.N = channels, states
        f32 = dict(dtype=torch.float32, device=device)
        self.dt_bias = nn.Parameter(torch.zeros(channels, **f32))
        self.A_log = nn.Parameter(torch.zeros(channels, states, **f32))
        self.D = nn.Parameter(torch.zeros(channels, **f32))

    def finalize(self):
        pass

    def state_shapes(self):
        return {"state": ((self.C, self.N), torch.float32)}

    def forward(self, x, dt_raw, z, B, C, state):
        dt, A = F.softplus(dt_raw.float() + self.dt_bias), -torch.exp(self.A_log)
        xf, B, C = x.float(), B.float(), C.float()
        y = torch.zeros(x.shape, dtype=torch.float32, device=x.device)
        for b, slot, r0, nq, start in _spans(_ctx()):
            S = state[slot].clone() if start > 0 else torch.zeros_like(state[slot])
            for t in range(r0, r0 + nq):
                S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * xf[t])[:, None] * B[t][None, :]
                y[t] = S @ C[t]
            state[slot] = S
        return ((y + self.D * xf) * F.silu(z.float())).to(x.dtype)


def _blended(dims, base, scaling):
    """(frequencies, magnitude of cos and sin)."""
    if not scaling:
        return torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float32), 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])
    edge = [dims * math.log(original / (2 * math.pi * float(scaling[k]))) / (2 * math.log(base)) for k in ("fast", "slow")]
    lo, hi = max(math.floor(edge[0]), 0), min(math.ceil(edge[1]), dims - 1)
    out = []
    for i in range(dims // 2):
        f, r = float(base) ** (-2.0 * i / dims), min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1.0 - r))
    return torch.tensor(out, dtype=torch.float32), 0.1 * math.log(factor) + 1.0


class RowNormAttention(nn.Module):
    def __init__(self, num_heads, num_kv_heads, head_dim, v_head_dim, scale, eps, rot_dims=0, rot_base=10000.0, rot_scaling=None,
                 device=None):
        super().__init__()
        self.H, self.G, self.D, self.Dv = num_heads, num_kv_heads, head_dim, v_head_dim
        self.scale, self.eps, self.rot_dims = float(scale), float(eps), int(rot_dims)
        f32 = dict(dtype=torch.float32, device=device)
        self.q_norm = nn.Parameter(torch.ones(num_heads * head_dim, **f32))
        self.k_norm = nn.Parameter(torch.ones(num_kv_heads * head_dim, **f32))
        freq, self.mag = _blended(rot_dims, rot_base, rot_scaling) if rot_dims else (None, 1.0)
        self.register_buffer("freq", freq.to(device) if freq is not None else None, persistent=False)

    def _prepare(self, x, weight, positions):
        T, n, D = x.shape
        x = (_unit_rms(x.float().reshape(T, n * D), self.eps) * weight).view(T, n, D)
        if self.rot_dims:
            turned = _turn(x, positions, self.freq, self.rot_dims)
            x = torch.cat([turned[..., :self.rot_dims] * self.mag, x[..., self.rot_dims:]], dim=-1)
        return x

    def forward(self, q, k, v, positions, k_cache, v_cache):
        ctx = _ctx()
        dt, T, H, G, D, Dv = q.dtype, q.shape[0], self.H, self.G, self.D, self.Dv
        qn, kn = self._prepare(q, self.q_norm, positions).to(dt), self._prepare(k, self.k_norm, positions).to(dt)
        bs = k_cache.shape[1]
        slots = ctx.slot_mapping.long()
        k_cache.view(-1, G, D)[slots] = kn
        v_cache.view(-1, G, Dv)[slots] = v
        cu_q, cu_k = ctx.cu_seqlens_q.tolist(), ctx.cu_seqlens_k.tolist()
        out = torch.zeros(T, H, Dv, dtype=torch.float32, device=q.device)
        for b in range(len(cu_q) - 1):
            nq, nk = cu_q[b + 1] - cu_q[b], cu_k[b + 1] - cu_k[b]
            if nq == 0:
                continue
            pos_k = torch.arange(nk, device=q.device)
            rows = ctx.block_tables[b].long()[pos_k // bs] * bs + pos_k % bs
            kk, vv = k_cache.view(-1, G, D)[rows].float(), v_cache.view(-1, G, Dv)[rows].float()
            vis = pos_k[None, :] <= nk - nq + torch.arange(nq, device=q.device)[:, None]
            qq = qn[cu_q[b]:cu_q[b + 1]].float()
            for h in range(H):
                g = h // (H // G)
                s = (qq[:, h] @ kk[:, g].t() * self.scale).masked_fill(~vis, float("-inf"))
                out[cu_q[b]:cu_q[b + 1], h] = torch.softmax(s, dim=-1) @ vv[:, g]
        return out.reshape(T, H * Dv).to(dt)


class FixedDecayMemory(nn.Module):
    def __init__(self, num_heads, key_dim, value_dim, decay, device=None):
        super().__init__()
        self.H, self.Dk, self.Dv = num_heads, key_dim, value_dim
        self.register_buffer("decay", torch.tensor([float(x) for x in decay], dtype=torch.float32, device=device), persistent=False)

    def state_shapes(self):
        return {"state": ((self.H, self.Dk, self.Dv), torch.float32)}

    def forward(self, q, k, v, cache):
        T = q.shape[0]
        act = lambda t: F.silu(t.float())
        q, k, v = act(q), act(k), act(v)
        out = torch.zeros(T, self.H, self.Dv, dtype=torch.float32, device=q.device)
        S_all = cache["state"]
        for b, slot, r0, nq, start in _spans(_ctx()):
            S = S_all[slot].clone() if start > 0 else torch.zeros_like(S_all[slot])
            for t in range(r0, r0 + nq):
                S = self.decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
                out[t] = (S * q[t][:, :, None]).sum(1)
            S_all[slot] = S
        return out.reshape(T, self.H * self.Dv)


class JoinGated(nn.Module):
    def __init__(self, mem_cols, eps, left_scale, right_scale, device=None):
        super().__init__()
        self.eps, self.left_scale, self.right_scale = float(eps), float(left_scale), float(right_scale)
        self.norm_weight = nn.Parameter(torch.ones(mem_cols, dtype=torch.float32, device=device))

    def forward(self, attn, head_gate, mem, gate):
        T, H = head_gate.shape
        left = attn.float().view(T, H, -1) * torch.sigmoid(head_gate.float())[:, :, None] * self.left_scale
        right = _unit_rms(mem, self.eps) * self.norm_weight * torch.sigmoid(gate.float()) * self.right_scale
        return torch.cat([left.reshape(T, -1), right], dim=1).to(attn.dtype)


class ClampedGLU(nn.Module):
    def __init__(self, limit, alpha=1.702, shift=1.0):
        super().__init__()
        self.limit, self.alpha, self.shift = float(limit), float(alpha), float(shift)

    def forward(self, x):
        g, u = x.float().chunk(2, dim=1)
        g, u = g.clamp(max=self.limit), u.clamp(-self.limit, self.limit)
        return (g * torch.sigmoid(self.alpha * g) * (u + self.shift)).to(x.dtype)


class ScaledSoftcap(nn.Module):
    def __init__(self, scale, cap):
        super().__init__()
        self.scale, self.cap = float(scale), float(cap)

    def forward(self, x):
        z = x.float() * self.scale
        return self.cap * torch.tanh(z / self.cap) if self.cap else z
