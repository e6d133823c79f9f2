#!/usr/bin/env python3
"""Tiralix beside its closest existing models with full-size records (Tutedra: recurrent and attention mixers behind a stream
boundary with scaled columns; Buvalix: a dense gated feed-forward, norms on sublayer outputs) at equal sizes, random weights:
every kernel of the design next to the like kernel, with its HBM or MFMA rate, and prefill / decode throughput of whole models
through the engine.  `python bench.py --tiralix` prints the record as one JSON line.  Every step names itself on stderr before
it uses the GPU."""
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
from nanovllm_amd.layers import gated_memory, linear_memory, row_norm_attention, tied_attention  # noqa: E402
from nanovllm_amd.model.tiralix import TiralixConfig, TiralixForCausalLM  # noqa: E402
from tools.buvalix_bench import buvalix_config, paged, random_buvalix, rate, timed  # noqa: E402
from tools.tutedra_bench import random_tutedra, tutedra_config  # noqa: E402


def note(what):
    print("tiralix_bench: " + what, file=sys.stderr, flush=True)


def both(rec, name, fn, like, like_fn, kw, like_kw, iters=20):
    """Times the two sides in turn, twice each, and keeps the better time of each side."""
    a, b = timed(fn, iters), timed(like_fn, iters)
    a, b = min(a, timed(fn, iters)), min(b, timed(like_fn, iters))
    rec[name], rec["like: " + like] = rate(a, **kw), rate(b, **like_kw)
    return a, b


def kernel_records(dev):
    out = {}
    bf = torch.bfloat16
    g = torch.Generator(device=dev).manual_seed(0)
    rn = lambda *s, dtype=bf: torch.randn(*s, generator=g, device=dev).to(dtype)
    W, bs, ff = 2048, 256, 4096
    for name, T in (("prefill_8192_tokens", 8192), ("decode_256_tokens", 256)):
        note("stream kernels, " + name)
        rec = {}
        x, a, w, ls = rn(T, W, dtype=torch.float32), rn(T, W), rn(W, dtype=torch.float32), rn(W, dtype=torch.float32)
        both(rec, "stream_boundary (normed and scaled output -> stream, copy in bf16)",
             lambda: ops.stream_boundary(x, normed=a, normed_weight=w, eps=1e-5, copy_dtype=bf),
             "stream_boundary_scaled (Tutedra: scaled output -> stream -> norm in bf16)",
             lambda: ops.stream_boundary_scaled(x, add=a, col_scale=ls, norm=w, eps=1e-5, out_dtype=bf),
             dict(nbytes=T * W * 12), dict(nbytes=T * W * 12))
        y = rn(T, 2 * ff)
        both(rec, "clamped_glu_rows (ff 4096)", lambda: ops.clamped_glu_rows(y, 7.0, 1.702, 1.0), "gelu_tanh_and_mul (ff 4096)",
             lambda: ops.gelu_tanh_and_mul(y), dict(nbytes=T * ff * 6), dict(nbytes=T * ff * 6))
        attn, hg, mem, gate = rn(T, W), rn(T, 16), rn(T, W, dtype=torch.float32), rn(T, W)
        both(rec, "join_gated (16 heads of 128 beside a memory of 2048 columns)",
             lambda: ops.join_gated(attn, hg, 0.7, mem, w, gate, 1e-5, 1.2), "stream_boundary_scaled (a norm over a row, as above)",
             lambda: ops.stream_boundary_scaled(x, add=a, col_scale=ls, norm=w, eps=1e-5, out_dtype=bf),
             dict(nbytes=T * W * (2 + 4 + 2 + 4)), dict(nbytes=T * W * 12))
        rows = min(T, 256)
        lg = rn(rows, 32000)
        both(rec, "scale_softcap (%d rows, vocabulary 32000)" % rows, lambda: ops.scale_softcap(lg, 0.5, 30.0),
             "torch: widened and scaled, no cap (Benarax)", lambda: lg.float() * 0.5, dict(nbytes=rows * 32000 * 6),
             dict(nbytes=rows * 32000 * 6))
        out[name] = rec

    inner, N, H, D = 4096, 16, 16, 128
    cases = {"prefill_4x2048": [2048] * 4, "prefill_1x8192": [8192], "chunk_1x512": [512], "decode_256_seqs": [1] * 256,
             "decode_32_seqs": [1] * 32}
    for name, n_qs in cases.items():
        note("recurrent kernels, " + name)
        ctx, pos, _ = paged(n_qs, [n + 100 for n in n_qs], bs, dev)
        ctx.num_leading_decode = sum(n == 1 for n in n_qs)                 # (the lists lead with their single tokens)
        ctx.portion_kinds = ops.portion_kinds(n_qs[ctx.num_leading_decode:])
        T, B = sum(n_qs), len(n_qs)
        nv.set_context(ctx)
        rec = {}
        q, k, v = rn(T, H, D), rn(T, H, D), rn(T, H, D)
        cache = {"state": torch.zeros(B, H, D, D, device=dev)}
        mem = gated_memory.FixedDecayMemory(H, D, D, [1.0 - 2.0 ** (-3 - 0.5 * h) for h in range(H)], device=dev)
        like = gated_memory.GatedWriteMemory(H, D, D, 1e-5, device=dev)
        spec = dict(nbytes=T * H * D * 8 + 2 * B * H * D * D * 4)
        ta, tb = both(rec, "fixed_decay_memory (16 heads 128 x 128, fp32 out)", lambda: mem(q, k, v, cache),
                      "gated_write_memory (Tutedra, 16 heads 128 x 128)", lambda: like(q, k, v, cache),
                      dict(nbytes=T * H * D * 10 + 2 * B * H * D * D * 4), spec, iters=5)
        rec["fixed_decay tokens/s, like"] = [round(T / ta), round(T / tb)]
        for n in (N, 64):
            scan = linear_memory.SelectiveScan(inner, n, device=dev)
            with torch.no_grad():
                scan.A_log.copy_(torch.log(torch.arange(1, n + 1, device=dev).float()).expand(inner, n))
                scan.dt_bias.fill_(-4.0)
            scan.finalize()
            st = torch.zeros(B, inner, n, device=dev)
            x, dtr, z, bc = rn(T, inner), rn(T, inner), rn(T, inner), rn(T, 128 + 2 * n)
            Bm, Cm = bc[:, 128:128 + n], bc[:, 128 + n:]
            ta, tb = both(rec, "selective_scan (%d channels x %d states)" % (inner, n), lambda: scan(x, dtr, z, Bm, Cm, st),
                          "gated_write_memory again", lambda: like(q, k, v, cache),
                          dict(nbytes=T * (inner * 8 + 4 * n) + 2 * B * inner * n * 4), spec, iters=5)
            rec["selective_scan (%d) state updates/s in 10^12, like" % n] = [round(T * inner * n / ta / 1e12, 3),
                                                                            round(T * H * D * D / tb / 1e12, 3)]
        conv = linear_memory.ConvBiasSilu(inner, 4, device=dev)
        xb, cs = rn(T, 2 * inner), torch.zeros(B, 3, inner, device=dev, dtype=bf)
        conv0 = tied_attention.ShortConv(inner, 4, device=dev)
        both(rec, "causal_conv_bias_silu (4096 channels, rows of the in-projection)", lambda: conv(xb[:, :inner], cs),
             "causal_conv without bias and activation (Tutedra)", lambda: conv0(xb[:, :inner], cs), dict(nbytes=T * inner * 4),
             dict(nbytes=T * inner * 4))
        nv.set_context(None)
        out["recurrent " + name] = rec

    Hq, G = 16, 8
    acases = {"prefill_4x2048": ([2048] * 4, [2048] * 4), "chunk_512_over_8192": ([512], [8192]),
              "decode_256_seqs_ctx_513_768": ([1] * 256, torch.randint(513, 769, (256,), generator=torch.Generator().manual_seed(1)).tolist()),
              "decode_8_seqs_ctx_8192": ([1] * 8, [8192] * 8)}
    for name, (n_qs, n_ks) in acases.items():
        for Dh, Dv in ((128, 128), (64, 128)):
            note("attention kernels %d/%d, %s" % (Dh, Dv, name))
            ctx, pos, nb = paged(n_qs, n_ks, bs, dev)
            T = sum(n_qs)
            nv.set_context(ctx)
            rec = {}
            rot = {"factor": 8.0, "original": 2048, "fast": 32.0, "slow": 1.0}
            att = row_norm_attention.RowNormAttention(Hq, G, Dh, Dv, Dh ** -0.5, 1e-5, Dh // 2, 1e4, rot, device=dev)
            old = tied_attention.KeyTiedAttention(Hq, G, Dh, Dh ** -0.5, 1e-5, Dh // 2, 1e4, None, device=dev)
            q, k, v = rn(T, Hq, Dh), rn(T, G, Dh), rn(T, G, Dv)
            kc, vc, vk = rn(nb, bs, G, Dh), rn(nb, bs, G, Dv), rn(nb, bs, G, Dh)
            both(rec, "row_norm_rope_store (whole-row norms, rotary on half, keys and values scattered)",
                 lambda: ops.row_norm_rope_store(pos, q, k, v, att.q_norm, att.k_norm, 1e-5, att.freq, Dh // 2, att.mag,
                                                 ctx.slot_mapping, kc, vc),
                 "head_norm_rope_store (Tutedra: per-head norms, prepared and raw keys scattered)",
                 lambda: ops.head_norm_rope_store(pos, q, k, old.q_norm, old.k_norm, 1e-5, old.freq, Dh // 2, ctx.slot_mapping, kc, vk),
                 dict(nbytes=T * (2 * (Hq + G) * Dh + 2 * G * Dv) * 2), dict(nbytes=T * (2 * Hq + 3 * G) * Dh * 2))
            full = sum(nq * (nk - nq) + nq * (nq + 1) // 2 for nq, nk in zip(n_qs, n_ks))
            singles = int(max(n_qs) == 1)
            t = timed(lambda: ops.attn_scoremod_paged(q, kc, vc, ctx.cu_seqlens_q, ctx.cu_seqlens_k, ctx.block_tables, Dh ** -0.5, 0.0,
                                                      None, None, max(n_qs), max(n_ks), singles), iters=5)
            rec["attention (the like kernel itself: attn_scoremod with every modifier off)"] = rate(
                t, nbytes=(sum(n_ks) * G * (Dh + Dv) * 2 + T * Hq * (Dh + Dv) * 2) if singles else None,
                flops=None if singles else 2 * (Dh + Dv) * Hq * full)
            nv.set_context(None)
            out["attention %d/%d %s" % (Dh, Dv, name)] = rec
    return out


def tiralix_config(width, n_groups, vocab, ff):
    left = {"heads": 16, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "rot": {"dims": 64, "base": 1e4, "scaling": {"factor": 8.0, "original": 2048, "fast": 32.0, "slow": 1.0}}}
    right = {"heads": 16, "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-3 - 0.5 * h) for h in range(16)]}
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
    group = [{"type": "mamba1", "mlp": mlp, "mixer": {"inner": 2 * width, "state": 16, "dt_rank": width // 16, "conv": 4}},
             {"type": "parallel", "mlp": mlp, "mixer": {"left": left, "right": right, "left_scale": 0.7, "right_scale": 0.7}}]
    return {"architecture": "Tiralix", "layers": group * (2 * n_groups), "norm": {"eps": 1e-5}, "vocab": vocab, "width": width,
            "logit_scale": 0.5, "logit_softcap": 30.0}


def like_tutedra_config(width, n_groups, vocab, ff):
    """Tutedra's recurrences and attention with its dense two-matrix feed-forward at the same number of weights."""
    cfg = tutedra_config(width, n_groups, vocab)
    for layer in cfg["layers"]:
        layer["mlp"] = {"kind": "dense", "ff": ff * 3 // 2}
    return cfg


def random_tiralix(cfg_dict, dev, dtype):
    cfg = TiralixConfig.from_dict(cfg_dict)
    model = TiralixForCausalLM(cfg, dtype=dtype, device=dev)
    g = torch.Generator(device=dev).manual_seed(0)
    with torch.no_grad():
        for name, p in model.named_parameters():
            if "norm" in name or name.endswith("scan.D"):
                p.fill_(1.0)
            elif name.endswith("dt_bias"):
                p.fill_(-4.0)
            elif name.endswith("A_log"):
                p.copy_(torch.log(torch.arange(1, p.shape[1] + 1, device=dev).float()).expand(p.shape))
            elif name.endswith("conv.bias"):
                p.zero_()
            else:
                p.copy_((torch.randn(p.shape, generator=g, device=dev) * (0.5 if "conv" in name else 0.02)).to(p.dtype))
    return model.finalize(), cfg


def model_records(dev, width=2048, n_groups=2, vocab=32000, prompt_len=1024, out_len=64, ff=6144):
    out = {"shape": dict(width=width, layers=4 * n_groups, vocab=vocab, prompt_len=prompt_len, out_len=out_len, block_size=256, ff=ff,
                         tiralix="mamba1 (4096 channels x 16 states) / parallel (16/8 heads of 128 beside 16 heads 128 x 128), dense gated ff",
                         tutedra="mlstm / attention / hgrn2 / attention, 16 heads of 128, dense ff of the same weights",
                         buvalix="channel_delta / attention / channel_delta / attention_2, 16 heads of 128, dense gated ff")}
    g = torch.Generator().manual_seed(0)

    def measure(made, batch, prompt_len):
        model, cfg = made
        prompts = [torch.randint(0, vocab, (prompt_len,), generator=g).tolist() for _ in range(batch)]
        warm = [torch.randint(0, vocab, (prompt_len,), generator=g).tolist() for _ in range(2)]
        eng = LLMEngine(model, cfg, block_size=256, num_kvcache_blocks=max(batch, 2) * (-(-(prompt_len + out_len) // 256)) + 8,
                        max_num_batched_tokens=8192, device=dev, eos=-1, max_num_seqs=max(batch, 2), long_prefill_token_threshold=0)
        eng.generate(warm, SamplingParams(0.0, 4))
        torch.cuda.synchronize()
        _, m = eng.generate(prompts, SamplingParams(0.0, out_len))
        s = m.summary()
        prefill = sum(t for t, _, only in m.step_times if not only)
        return {"prefill_tok_per_s": round(batch * prompt_len / prefill), "decode_tok_per_s": round(s["decode_only_tok_per_s"]),
                "mean_tpot_ms": round(s["mean_tpot_ms"], 3), "output_tok_per_s": round(s["output_tok_per_s"])}

    bf = torch.bfloat16
    sides = {"tiralix": lambda: random_tiralix(tiralix_config(width, n_groups, vocab, ff), dev, bf),
             "like: tutedra": lambda: random_tutedra(like_tutedra_config(width, n_groups, vocab, ff), dev, bf),
             "like: buvalix": lambda: random_buvalix(buvalix_config(width, ff, n_groups, vocab), dev, bf)}
    for name, make in sides.items():
        made = make()
        for batch, plen in ((32, prompt_len), (128, prompt_len), (1, 8000)):
            note("model: %s, batch %d, prompts of %d" % (name, batch, plen))
            out.setdefault("batch %d, prompts of %d" % (batch, plen), {})[name] = measure(made, batch, plen)
        del made
        torch.cuda.empty_cache()
    return out


def run(device="cuda:0", kernels=True, models=True):
    rec = {"metric": "tiralix_vs_like_models", "rooflines": {"hbm_TB_s": 8.0, "mfma_bf16_PFLOP_s": 2.5},
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
