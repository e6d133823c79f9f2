#!/usr/bin/env python3
"""Nekodra beside Benarax (the closest existing model: latent attention over a paged latent cache, one norm that feeds mixer
and feed-forward side by side, routed experts) at equal sizes, random weights: every kernel of the design next to the like
kernel, with its HBM or MFMA rate, and prefill / decode throughput of whole models through the engine.
`python bench.py --nekodra` prints the record as one JSON line.  Every step names itself on stderr before it uses the GPU."""
import argparse
import json
import os
import sys

import torch

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, ROOT)
import nanovllm_amd as nv  # noqa: E402
from nanovllm_amd import ops  # noqa: E402
from nanovllm_amd.engine.llm_engine import LLMEngine  # noqa: E402
from nanovllm_amd.engine.sequence import SamplingParams  # noqa: E402
from nanovllm_amd.layers import latent_attention, moe  # noqa: E402
from nanovllm_amd.model.nekodra import NekodraConfig, NekodraForCausalLM  # noqa: E402
from tools.benarax_bench import random_benarax  # noqa: E402
from tools.buvalix_bench import paged, rate, timed  # noqa: E402


def note(what):
    print("nekodra_bench: " + what, file=sys.stderr, flush=True)


def both(rec, name, fn, like, like_fn, kw, like_kw, iters=20):
    """Times the two sides in turn, twice each, and keeps the better time of each side."""
    a, b = timed(fn, iters), timed(like_fn, iters)
    a, b = min(a, timed(fn, iters)), min(b, timed(like_fn, iters))
    rec[name], rec["like: " + like] = rate(a, **kw), rate(b, **like_kw)


def kernel_records(dev):
    out = {}
    bf = torch.bfloat16
    g = torch.Generator(device=dev).manual_seed(0)
    rn = lambda *s, dtype=bf: torch.randn(*s, generator=g, device=dev).to(dtype)
    W, bs, top = 2048, 256, 4
    for name, T in (("prefill_8192_tokens", 8192), ("decode_256_tokens", 256)):
        note("stream kernels, " + name)
        rec = {}
        x, a, b, parts = rn(T, W, dtype=torch.float32), rn(T, W), rn(T, W), rn(T, top, W, dtype=torch.float32)
        w, c = rn(W, dtype=torch.float32), rn(W, dtype=torch.float32)
        ids = torch.randint(0, 36, (T, top), generator=g, device=dev, dtype=torch.int32)
        wts = torch.rand(T, top, generator=g, device=dev)
        h = rn(T, W)
        n_prod = int((ids < 32).sum())
        n_thru = int((ids >= 32).any(dim=1).sum())
        both(rec, "stream_layernorm_pair (mixer + shared expert + routed parts -> stream -> two norms, bf16 + bf16 + fp32)",
             lambda: ops.stream_layernorm_pair(x, adds=[a, b], routed=(parts, ids, wts, 32, h), norm_a=(w, c), norm_b=(w, c), eps=1e-5,
                                               out_dtype=bf, want_f32_b=True),
             "stream_boundary (mixer + 4 expert parts -> stream -> grouped norm, fp32 + bf16)",
             lambda: ops.stream_boundary(x, add=a, add_parts=parts, mult=0.5, norm=w, groups=4, eps=1e-5, out_dtype=bf, want_f32=True),
             dict(nbytes=T * W * (8 + 4 + 8) + n_prod * W * 4 + n_thru * W * 2), dict(nbytes=T * W * (8 + 2 + 16 + 6)))
        y = rn(T, 8192)
        both(rec, "silu_and_mul_rows (ff 4096)", lambda: ops.silu_and_mul_rows(y), "gelu_tanh_and_mul (ff 4096)",
             lambda: ops.gelu_tanh_and_mul(y), dict(nbytes=T * 4096 * 6), dict(nbytes=T * 4096 * 6))
        ids64, pos = torch.randint(0, 32000, (T,), generator=g, device=dev), torch.arange(T, device=dev) % 2048
        table, ptab = rn(32000, W), rn(2048, W)
        both(rec, "embed_positions", lambda: ops.embed_positions(ids64, pos, table, ptab), "torch embedding, widened to fp32",
             lambda: torch.nn.functional.embedding(ids64, table).float(), dict(nbytes=T * W * 8), dict(nbytes=T * W * 6))
        out[name] = rec

    H = 16
    for rank, (lr, lR, dim, vdim) in ((160, (128, 32, 128, 96)), (256, (192, 64, 192, 128)), (512, (512, 64, 128, 128))):
        cases = {"prefill_4x2048": ([2048] * 4, [2048] * 4), "chunk_512_over_8192": ([512], [8192]),
                 "decode_256_seqs_ctx_513_768": ([1] * 256, torch.randint(513, 769, (256,), generator=torch.Generator().manual_seed(1)).tolist()),
                 "decode_32_seqs_ctx_1088": ([1] * 32, [1088] * 32), "decode_8_seqs_ctx_8192": ([1] * 8, [8192] * 8)}
        for name, (n_qs, n_ks) in cases.items():
            note("attention kernels, rank %d, %s" % (rank, name))
            ctx, pos, nb = paged(n_qs, n_ks, bs, dev)
            T = sum(n_qs)
            nv.set_context(ctx)
            rec = {}
            wl, lw = torch.ones(rank, device=dev), torch.ones(lr, device=dev)
            kc, kc2 = rn(nb, bs, 1, rank), rn(nb, bs, 1, lr + lR)
            ckv, ckv2 = rn(T, rank), rn(T, lr + lR)
            lat = latent_attention.LatentAttention(H, lr, lR, 0.1, 1e-5, 1e4, None, device=dev)
            q2, ql2 = rn(T, H, dim), rn(T, H, lr)
            both(rec, "latent_store", lambda: ops.latent_store(ckv, wl, ctx.slot_mapping, kc, 1e-5),
                 "latent_prep_store (also rotates and assembles the queries)",
                 lambda: ops.latent_prep_store(q2, ql2, ckv2, lw, lat.freq, lat.mag, True, pos, ctx.slot_mapping, kc2, kc2[..., :lr], lR, 1e-5),
                 dict(nbytes=T * rank * 4), dict(nbytes=T * (H * (lr + lR) * 4 + (lr + lR) * 4)))
            q, gate, sink = rn(T, H * dim + H * vdim), rn(T, H * vdim), torch.zeros(H, device=dev)
            uk, uv = rn(H, rank, dim), rn(H, vdim, rank)
            uk2, uv2 = rn(H, dim, rank), rn(H, rank, vdim)
            qv = q[:, :H * dim]
            both(rec, "head_linear, key up-projection on the query", lambda: ops.head_linear(qv, uk),
                 "torch.bmm (result per head, before any transposed copy)",
                 lambda: torch.bmm(qv.view(T, H, dim).transpose(0, 1), uk2),
                 dict(nbytes=T * H * (dim + rank) * 2, flops=2 * T * H * dim * rank), dict(nbytes=T * H * (dim + rank) * 2, flops=2 * T * H * dim * rank))
            ol = rn(T, H * rank)
            both(rec, "head_linear, value up-projection with the sigmoid gate", lambda: ops.head_linear(ol, uv, gate),
                 "torch.bmm, transposed copy (no gate)",
                 lambda: torch.bmm(ol.view(T, H, rank).transpose(0, 1), uv2).transpose(0, 1).reshape(T, -1),
                 dict(nbytes=T * H * (rank + 2 * vdim) * 2, flops=2 * T * H * vdim * rank),
                 dict(nbytes=T * H * (rank + vdim) * 2, flops=2 * T * H * vdim * rank))
            pairs = sum(nq * (nk - nq) + nq * (nq + 1) // 2 for nq, nk in zip(n_qs, n_ks))
            singles = int(max(n_qs) == 1)
            meta = (ctx.cu_seqlens_q, ctx.cu_seqlens_k, ctx.block_tables, 0.1)
            att = lambda qq, kk, vd, sk: ops.attn_latent_paged(qq, kk, kk[..., :vd], *meta, sk, max(n_qs), max(n_ks), singles)
            old = lambda qq, kk, vd, sk: ops.attn_scoremod_paged(qq, kk, kk[..., :vd], *meta, 0.0, sk, None, max(n_qs), max(n_ks), singles)
            qa, qb = rn(T, H, rank), rn(T, H, lr + lR)
            spec = lambda d, v: dict(nbytes=sum(n_ks) * d * 2 + T * H * (d + v) * 2 if singles else None, flops=2 * (d + v) * H * pairs)
            both(rec, "latent attention with a sink (key %d, value %d)" % (rank, rank), lambda: att(qa, kc, rank, sink),
                 "Benarax latent attention (key %d, value %d)" % (lr + lR, lr), lambda: att(qb, kc2, lr, None), spec(rank, rank),
                 spec(lr + lR, lr), iters=10)
            rec["like: the general paged attention launch on the same rows"] = rate(timed(lambda: old(qa, kc, rank, sink), 5), **spec(rank, rank))
            nv.set_context(None)
            out["attention rank %d, %s" % (rank, name)] = rec

    E, idn, ff = 32, 4, 1024
    gu, dn = rn(E, 2 * ff, W) * 0.02, rn(E, W, ff) * 0.02
    router, ex, like = moe.SoftmaxRouter(E + idn, top, 2.0, device=dev), moe.SiluExperts(), moe.MoEExperts(top, 7.0)
    plain = moe.SoftmaxRouter(E, top, 2.0, device=dev)
    for name, T in (("prefill_8192_tokens", 8192), ("decode_256_tokens", 256), ("decode_32_tokens", 32)):
        note("expert kernels, " + name)
        h, lg, lg2 = rn(T, W), rn(T, E + idn, dtype=torch.float32), rn(T, E, dtype=torch.float32)
        rec = {"moe_route_softmax (32 + 4 experts, top 4)": rate(timed(lambda: router(lg)), nbytes=T * ((E + idn) * 4 + top * 8))}
        spec = dict(flops=2 * T * top * 3 * ff * W, nbytes=min(E, T * top) * 3 * ff * W * 2 + T * W * (2 + 4 * top))

        def routed():
            i, w = plain(lg2)
            return ex(h, i, w, gu, dn)
        both(rec, "softmax router + SiLU experts (32 experts, top 4, ff 1024)", routed,
             "routed clamped-GLU experts behind a softmax over the chosen", lambda: like(h, lg2, gu, dn), spec, spec, iters=5)
        out["feed-forward " + name] = rec
    return out


def nekodra_config(width, layers, vocab, share=True, rank=160, identity=4, shared=True, positions=4096):
    mlp = {"kind": "moe", "expert": {"ff": 1024}, "router": {"experts": 32, "identity": identity, "top": 4, "scale": 2.0}}
    if shared:
        mlp["shared"] = {"ff": 1024}
    mix = {"heads": 16, "dim": 128, "vdim": 96, "kv_rank": rank, "scale": 128 ** -0.5}
    ls = [{"type": "latent_attention", "mlp": mlp, "mixer": dict(mix, kv_from=i - 1) if share and i % 2 else mix} for i in range(layers)]
    return {"architecture": "Nekodra", "layers": ls, "norm": {"eps": 1e-5}, "vocab": vocab, "width": width, "max_positions": positions}


def like_config(width, layers, vocab):
    """Benarax with latent attention in every layer and none of its optional parts, at the same sizes."""
    mlp = {"kind": "moe", "router": {"experts": 32, "top": 4}, "expert": {"ff": 1024, "limit": 7.0}}
    lat = {"heads": 16, "dim": 96, "rot_dim": 32, "vdim": 96, "q_rank": 768, "kv_rank": 128, "scale": 128 ** -0.5,
           "rot": {"dims": 32, "base": 1e4}}
    return {"architecture": "Benarax", "layers": [{"type": "latent_attention", "mlp": mlp, "mixer": lat}] * layers,
            "norm": {"eps": 1e-5, "groups": 1}, "vocab": vocab, "width": width}


def random_nekodra(cfg_dict, dev, dtype):
    cfg = NekodraConfig.from_dict(cfg_dict)
    model = NekodraForCausalLM(cfg, dtype=dtype, device=dev)
    g = torch.Generator(device=dev).manual_seed(0)
    with torch.no_grad():
        for name, p in model.named_parameters():
            if "norm" in name and not name.endswith("bias"):
                p.fill_(1.0)
            else:
                p.copy_((torch.randn(p.shape, generator=g, device=dev) * (0.02 if p.dim() > 1 else 0.01)).to(p.dtype))
    return model.finalize(), cfg


def model_records(dev, width=2048, layers=8, vocab=32000, prompt_len=1024, out_len=64):
    out = {"shape": dict(width=width, layers=layers, vocab=vocab, prompt_len=prompt_len, out_len=out_len, block_size=256,
                         nekodra="16 heads, latent 160, value 96; 32 experts of ff 1024 (and 4 identity experts), top 4, shared expert ff 1024",
                         benarax="latent attention in every layer: 16 heads, latent 128 + 32, value 96; 32 experts of ff 1024, top 4; no "
                                 "input convolution, no token table")}
    g = torch.Generator().manual_seed(0)

    def measure(make, batch):
        model, cfg = make
        prompts = [torch.randint(0, vocab, (prompt_len,), generator=g).tolist() for _ in range(batch)]
        warm = [torch.randint(0, vocab, (prompt_len,), generator=g).tolist() for _ in range(2)]
        eng = LLMEngine(model, cfg, block_size=256, num_kvcache_blocks=batch * (-(-(prompt_len + out_len) // 256)) + 8,
                        max_num_batched_tokens=8192, device=dev, eos=-1, max_num_seqs=batch, long_prefill_token_threshold=0)
        eng.generate(warm, SamplingParams(0.0, 4))
        torch.cuda.synchronize()
        _, m = eng.generate(prompts, SamplingParams(0.0, out_len))
        s = m.summary()
        prefill = sum(t for t, _, only in m.step_times if not only)
        return {"prefill_tok_per_s": round(batch * prompt_len / prefill), "decode_tok_per_s": round(s["decode_only_tok_per_s"]),
                "mean_tpot_ms": round(s["mean_tpot_ms"], 3), "output_tok_per_s": round(s["output_tok_per_s"])}

    sides = {"nekodra, every second layer on the latents of the one before": lambda: random_nekodra(nekodra_config(width, layers, vocab), dev, torch.bfloat16),
             "nekodra at the like model's parts (own latents, no shared or identity experts)":
                 lambda: random_nekodra(nekodra_config(width, layers, vocab, share=False, identity=0, shared=False), dev, torch.bfloat16),
             "like: benarax": lambda: random_benarax(like_config(width, layers, vocab), dev, torch.bfloat16)}
    for name, make in sides.items():
        built = make()
        for batch in (32, 128):
            note("model: %s, batch %d" % (name, batch))
            out.setdefault("batch %d" % batch, {})[name] = measure(built, batch)
        del built
        torch.cuda.empty_cache()
    return out


def run(device="cuda:0", kernels=True, models=True):
    rec = {"metric": "nekodra_vs_like_model", "rooflines": {"hbm_TB_s": 8.0, "mfma_bf16_PFLOP_s": 2.5},
           "data": "synthetic", "dtype": "bf16"}
    if kernels:
        rec["kernels"] = kernel_records(device)
    if models:
        rec["models"] = model_records(device)
    return rec


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--no-kernels", action="store_true")
    ap.add_argument("--no-models", action="store_true")
    a = ap.parse_args()
    print(json.dumps(run(kernels=not a.no_kernels, models=not a.no_models)))
