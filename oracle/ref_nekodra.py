"""Oracle (test infrastructure): a plain, slow restatement of the Nekodra design, one function per mechanism,
whole sequences at a time, no cache and no batching.  It shares nothing with the product path: tests compare
the engine (paged latent cache, chunked prompts, mixed batches, HIP kernels) with these functions.

`dtype=torch.float32` computes everything in 32-bit.  With `torch.bfloat16` the matrix products take bfloat16
operands (fp32 accumulation, bfloat16 result), the cached latent is bfloat16, and everything the design keeps in
32-bit stays there: the residual stream, norms, attention scores and weights, router scores.

A model is (cfg, weights): cfg the parsed config.json, weights a dict name -> tensor as stored.

The design in short.  x_0 = embed[token] + pos[position].  Every layer reads the stream through two layer norms with
biases, side by side:  x += mixer(norm1(x)) + ff(norm2(x)).  The mixer is latent attention without positions: keys and
values are per-head projections of one RMS-normed low-rank latent per token, a learned sink joins every head's softmax
denominator, and the heads' outputs are gated by sigmoid(W_g h) in front of the output projection.  A layer may read
the latents of an earlier layer instead of having its own.  The feed-forward is a mixture of SiLU-gated experts chosen
by biased softmax scores, some of which hand their input through unchanged, plus a shared expert.
logits = head layernorm(x).
"""
from __future__ import annotations

import torch
import torch.nn.functional as F


def linear(x, w, dtype=torch.float32):
    return F.linear(x.to(dtype), w.to(dtype))


def layer_norm(x, w, b, eps):
    x = x.float()
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w.float() + b.float()


def rms_unit(x, eps):
    x = x.float()
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def embed(w, tokens):
    n = len(tokens)
    return w["embed"][torch.tensor(tokens)].float() + w["pos"][:n].float()


# ------------------------------------------------------------------------------------------ mixer
def latents(w, p, h, eps, dtype):
    """The row a token leaves in the cache: its RMS-normed low-rank projection."""
    return (rms_unit(linear(h, w[p + "dkv"], dtype), eps) * w[p + "dkv.norm"].float()).to(dtype)


def sink_softmax(s, sink):
    """Rows of s as exp(s_j) / (exp(sink) + sum_j exp(s_j)); -inf entries weigh nothing."""
    m = torch.maximum(s.max(-1, keepdim=True).values, sink.float().reshape(1, 1))
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink.float() - m))


def latent_attention(m, w, p, h, c, dtype):
    """h [T, W] the mixer's input, c [T, rank] the latents it reads (its own or another layer's)."""
    T = h.shape[0]
    H, D, Dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = linear(h, w[p + "q"], dtype).float().view(T, H, D)
    k = linear(c, w[p + "uk"], dtype).float().view(T, H, D)
    v = linear(c, w[p + "uv"], dtype).float().view(T, H, Dv)
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, H, Dv)
    for i in range(H):
        s = (q[:, i] @ k[:, i].t()) * float(m["scale"])
        out[:, i] = sink_softmax(s.masked_fill(hidden, float("-inf")), w[p + "sink"][i]) @ v[:, i]
    o = out.reshape(T, H * Dv).to(dtype).float() * torch.sigmoid(linear(h, w[p + "g"], dtype).float())
    return linear(o.to(dtype), w[p + "o"], dtype)


# ------------------------------------------------------------------------------------------ feed-forward
def gated_unit(w, p, h, dtype):
    """down(silu(gate h) * (up h))."""
    g, u = linear(h, w[p + "gate"], dtype).float(), linear(h, w[p + "up"], dtype).float()
    return linear((g * torch.sigmoid(g) * u).to(dtype), w[p + "down"], dtype).float()


def route(mlp, w, p, h32):
    """(chosen experts [T, top], their weights [T, top]): softmax scores over all experts, identity experts included
    (they are the last ones); the choice adds a per-expert correction, the weights are the plain scores of the chosen
    times a constant, not renormalised."""
    r = mlp["router"]
    s = torch.softmax(F.linear(h32.float(), w[p + "router"].float()), dim=-1)
    choice = s + w[p + "correction"].float() if p + "correction" in w else s
    ids = choice.topk(int(r["top"]), dim=-1).indices
    return ids, s.gather(1, ids) * float(r.get("scale", 1.0))


def moe(mlp, w, p, h32, dtype):
    h = h32.to(dtype)
    E = int(mlp["router"]["experts"])
    ids, weights = route(mlp, w, p, h32)
    out = torch.zeros(h32.shape)
    for t in range(h.shape[0]):
        for e, g in zip(ids[t].tolist(), weights[t].tolist()):
            y = gated_unit(w, f"{p}e{e}.", h[t:t + 1], dtype)[0] if e < E else h[t].float()
            out[t] += g * y
    if mlp.get("shared"):
        out = out + gated_unit(w, p + "shared.", h, dtype)
    return out


# ------------------------------------------------------------------------------------------ the model
def forward(cfg, weights, tokens, dtype=torch.float32):
    """Returns (logits [T, vocab] float32, the residual stream after every layer [layers, T, width])."""
    w, eps = weights, float(cfg["norm"]["eps"])
    x = embed(w, tokens)
    streams, cached = [], {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps).to(dtype)
        if m.get("kv_from") is None:
            cached[i] = latents(w, p + "mix.", h, eps, dtype)
        src = i if m.get("kv_from") is None else int(m["kv_from"])
        y = latent_attention(m, w, p + "mix.", h, cached[src], dtype).float()
        if L.get("mlp") is not None:
            y = y + moe(L["mlp"], w, p + "mlp.", layer_norm(x, w[p + "norm2"], w[p + "norm2.b"], eps), dtype)
        x = x + y
        streams.append(x.clone())
    logits = linear(layer_norm(x, w["final.norm"], w["final.norm.b"], eps).to(dtype), w["head"], dtype).float()
    return logits, torch.stack(streams)
