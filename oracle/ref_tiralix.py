"""Oracle (test infrastructure): a plain, slow restatement of the Tiralix design, one function per mechanism, whole
sequences at a time, no cache and no batching.  It shares nothing with the product path: tests compare the engine (paged
cache, state slots, chunked prompts, mixed batches, HIP kernels) with these functions.

`dtype=torch.float32` computes everything in 32-bit.  With `torch.bfloat16` the matrix products, the short convolution and
the activations around them take bfloat16 operands (fp32 accumulation, bfloat16 result) and everything the design keeps in
32-bit stays there: the residual stream, norms, rotary angles, attention scores and weights, and both recurrences with
their decays, step sizes, exponentials and states.

A model is (cfg, weights): cfg the parsed config.json, weights a dict name -> tensor as stored.

The design in short.  x_0 = embed[token].  The sublayers read the stream itself; each output is RMS-normed and scaled per
column on its way back in:
    x += ls1 * norm1(mixer(x));  x += ls2 * norm2(ff(x)).
The mixer is a selective scan (`mamba1`) or two mixers on the same input, added with one factor each (`parallel`): grouped-query
softmax attention with whole-row q / k norms, blended rotary frequencies and one sigmoid gate per head, beside a linear
attention with one fixed decay per head.  The feed-forward is a clamped gated unit.
logits = cap * tanh(logit_scale * (embed rmsnorm(x)) / cap).
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F


def linear(x, w, dtype=torch.float32):
    return F.linear(x.to(dtype), w.to(dtype))


def rms_norm(x, w, eps):
    x = x.float()
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.float()


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 20.0, z, torch.log1p(torch.exp(torch.clamp(z, max=20.0))))


# ------------------------------------------------------------------------------------------ rotary
def rotary_frequencies(rot):
    """(f_i, magnitude): f_i = base^(-2i/dims); with scaling, pairs in front of dim(fast) keep f, pairs behind dim(slow)
    take f / factor, those between a linear blend; cos and sin are multiplied by 0.1 ln(factor) + 1."""
    dims, base = int(rot["dims"]), float(rot["base"])
    sc = rot.get("scaling")
    mag = 1.0
    if sc:
        factor, original = float(sc["factor"]), float(sc["original"])
        at = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
        lo = max(math.floor(at(float(sc["fast"]))), 0)
        hi = min(math.ceil(at(float(sc["slow"]))), dims - 1)
        mag = 0.1 * math.log(factor) + 1.0
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / factor * ramp + f * (1.0 - ramp)
        out.append(f)
    return torch.tensor(out, dtype=torch.float32), mag


def rotate_halves(x, positions, freq, mag):
    """x [T, heads, D]: pair (i, i + len(freq)) turns by position * freq[i], both parts times mag; the rest passes."""
    half = freq.numel()
    x = x.float()
    out = x.clone()
    ang = positions.to(torch.float32)[:, None] * freq[None, :]
    c, s = (torch.cos(ang) * mag)[:, None, :], (torch.sin(ang) * mag)[:, None, :]
    a, b = x[..., :half], x[..., half:2 * half]
    out[..., :half] = a * c - b * s
    out[..., half:2 * half] = b * c + a * s
    return out


# ------------------------------------------------------------------------------------------ mixers
def softmax_attention(q, k, v, scale):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; causal; returns [T, H, Dv] float32."""
    T, H = q.shape[:2]
    G = k.shape[1]
    q, k, v = q.float(), k.float(), v.float()
    vis = torch.tril(torch.ones(T, T, dtype=torch.bool))
    out = torch.zeros(T, H, v.shape[2])
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t() * scale).masked_fill(~vis, float("-inf"))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (e / e.sum(-1, keepdim=True)) @ v[:, g]
    return out


def gated_attention(m, w, p, h, eps, dtype=torch.float32):
    """The left mixer: h [T, W] -> [T, W]."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = linear(h, w[p + "q"], dtype), linear(h, w[p + "k"], dtype), linear(h, w[p + "v"], dtype)
    q, k = rms_norm(q, w[p + "q.norm"], eps).view(T, H, D), rms_norm(k, w[p + "k.norm"], eps).view(T, G, D)
    if m.get("rot"):
        freq, mag = rotary_frequencies(m["rot"])
        pos = torch.arange(T)
        q, k = rotate_halves(q, pos, freq, mag), rotate_halves(k, pos, freq, mag)
    o = softmax_attention(q.to(dtype), k.to(dtype), v.view(T, G, Dv), m["scale"])
    gate = torch.sigmoid(linear(h, w[p + "g"], dtype).float())
    o = (o.to(dtype).float() * gate[:, :, None]).reshape(T, H * Dv)
    return linear(o, w[p + "o"], dtype)


def decayed_memory(q, k, v, decay):
    """q, k [T, H, D], v [T, H, Dv], decay [H]:  S <- decay S + k v^T;  o = S^T q (the write comes first)."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2])
    out = torch.zeros(T, H, v.shape[2])
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def lightning_attention(m, w, p, h, eps, dtype=torch.float32):
    """The right mixer: h [T, W] -> [T, W]."""
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    act = lambda n: silu(linear(h, w[p + n], dtype).float()).to(dtype).float()
    o = decayed_memory(act("q").view(T, H, D), act("k").view(T, H, D), act("v").view(T, H, Dv),
                       torch.tensor(m["decay"], dtype=torch.float32))
    o = rms_norm(o.reshape(T, H * Dv), w[p + "norm"], eps) * torch.sigmoid(linear(h, w[p + "g"], dtype).float())
    return linear(o, w[p + "o"], dtype)


def parallel_mixer(m, w, p, h, eps, dtype=torch.float32):
    left = gated_attention(m["left"], w, p + "left.", h, eps, dtype).float()
    right = lightning_attention(m["right"], w, p + "right.", h, eps, dtype).float()
    return m["left_scale"] * left + m["right_scale"] * right


def causal_conv_silu(x, w, b, dtype=torch.float32):
    """x [T, C], w [C, taps]: silu(b + sum_j w[:, j] x_(t - taps + 1 + j)), zeros before the start; result in dtype."""
    T, taps = x.shape[0], w.shape[1]
    x, w = x.float(), w.float()
    y = b.float().repeat(T, 1)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * x[s]
    return silu(y).to(dtype)


def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, I], A [I, N], B, C [T, N], D [I]:  S <- exp(dt A) S + dt x B;  y = S C + D x."""
    T, I = x.shape
    S = torch.zeros(I, A.shape[1])
    y = torch.zeros(T, I)
    for t in range(T):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = (S * C[t][None, :]).sum(1) + D * x[t]
    return y


def mamba_mixer(m, w, p, h, dtype=torch.float32):
    I, N, R = m["inner"], m["state"], m["dt_rank"]
    xz = linear(h, w[p + "in"], dtype)
    x, z = xz[:, :I], xz[:, I:]
    x = causal_conv_silu(x, w[p + "conv"], w[p + "conv.b"], dtype)
    dbc = linear(x, w[p + "x"], dtype)
    dt = softplus(linear(dbc[:, :R], w[p + "dt"], dtype).float() + w[p + "dt.b"].float())
    y = selective_scan(x.float(), dt, -torch.exp(w[p + "A_log"].float()), dbc[:, R:R + N].float(), dbc[:, R + N:].float(),
                       w[p + "D"].float())
    return linear(y * silu(z.float()), w[p + "o"], dtype)


# ------------------------------------------------------------------------------------------ feed-forward
def clamped_glu(g, u, limit, alpha=1.702):
    g, u = torch.clamp(g.float(), max=limit), torch.clamp(u.float(), -limit, limit)
    return g * torch.sigmoid(alpha * g) * (u + 1.0)


def feed_forward(m, w, p, x, dtype=torch.float32):
    if m["kind"] != "dense":
        raise ValueError(m["kind"])
    y = clamped_glu(linear(x, w[p + "gate"], dtype), linear(x, w[p + "up"], dtype), float(m["limit"]))
    return linear(y, w[p + "down"], dtype)


# ------------------------------------------------------------------------------------------ the whole model
def forward(cfg, w, tokens, dtype=torch.float32):
    """(logits [T, vocab], stream after every layer [layers, T, width]) in float32."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)].float()
    streams = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        if L["type"] == "parallel":
            y = parallel_mixer(L["mixer"], w, p + "mix.", x, eps, dtype)
        elif L["type"] == "mamba1":
            y = mamba_mixer(L["mixer"], w, p + "mix.", x, dtype)
        else:
            raise ValueError(L["type"])
        x = x + w[p + "ls1"].float() * rms_norm(y, w[p + "norm1"], eps)
        if L.get("mlp") is not None:
            x = x + w[p + "ls2"].float() * rms_norm(feed_forward(L["mlp"], w, p + "mlp.", x, dtype), w[p + "norm2"], eps)
        streams.append(x)
    z = linear(rms_norm(x, w["final.norm"], eps), w["embed"], dtype).float() * float(cfg["logit_scale"])
    cap = float(cfg.get("logit_softcap") or 0.0)
    return (cap * torch.tanh(z / cap) if cap else z), torch.stack(streams)
