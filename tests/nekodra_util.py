"""Helpers of the Nekodra tests: small configurations, random checkpoints in the design's tensor names, and engines on the
CPU stand-ins or on the HIP layers.  The replay driver and the error measures are shared with the other designs' tests."""
import math

import torch

import nanovllm_amd  # noqa: F401
from buvalix_util import paged_context, rel_err, replay  # noqa: F401
from nanovllm_amd.engine.llm_engine import LLMEngine
from nanovllm_amd.model.nekodra import NekodraConfig, NekodraForCausalLM
from oracle import ref_nekodra, ref_nekodra_modules


def moe(experts=5, identity=2, top=3, scale=1.75, ff=20, shared=28):
    m = {"kind": "moe", "router": {"experts": experts, "identity": identity, "top": top, "scale": scale}, "expert": {"ff": ff}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(heads=3, dim=10, vdim=14, rank=18, scale=None, kv_from=None, mlp="default"):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale or 1.3 / math.sqrt(dim)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": moe() if mlp == "default" else mlp}


def config(layers, vocab=83, width=36, eps=1e-5, positions=300):
    return {"architecture": "Nekodra", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width, "max_positions": positions}


def random_checkpoint(cfg: dict, seed: int, dtype=torch.bfloat16, correction=True) -> dict:
    """Tensors by checkpoint name, stored in bfloat16 like a file (so every dtype sees the same values)."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    rn = lambda *s, std=1.0, mean=0.0: (torch.randn(*s, generator=g) * std + mean).to(dtype)
    lin = lambda o, i, gain=1.0: rn(o, i, std=gain / math.sqrt(i))
    t = {"embed": rn(V, W), "pos": rn(cfg["max_positions"], W, std=0.5), "head": lin(V, W), "final.norm": rn(W, std=0.1, mean=1.0),
         "final.norm.b": rn(W, std=0.1)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, D, Dv, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        for n in ("norm1", "norm2") if L["mlp"] is not None else ("norm1",):
            t[p + n], t[p + n + ".b"] = rn(W, std=0.2, mean=1.0), rn(W, std=0.2)
        q = p + "mix."
        t[q + "q"], t[q + "g"], t[q + "o"] = lin(H * D, W, 2.0), lin(H * Dv, W, 2.0), lin(W, H * Dv)
        t[q + "uk"], t[q + "uv"], t[q + "sink"] = lin(H * D, R, 1.5), lin(H * Dv, R), rn(H, std=1.5)
        if m.get("kv_from") is None:
            t[q + "dkv"], t[q + "dkv.norm"] = lin(R, W), rn(R, std=0.2, mean=1.0)
        if L["mlp"] is None:
            continue
        q, r, ff = p + "mlp.", L["mlp"]["router"], L["mlp"]["expert"]["ff"]
        n = r["experts"] + r.get("identity", 0)
        t[q + "router"] = lin(n, W, 1.5)
        if correction:
            t[q + "correction"] = rn(n, std=0.1)
        units = [(f"e{e}.", ff) for e in range(r["experts"])] + ([("shared.", L["mlp"]["shared"]["ff"])] if L["mlp"].get("shared") else [])
        for u, f in units:
            t[q + u + "gate"], t[q + u + "up"], t[q + u + "down"] = lin(f, W, 1.5), lin(f, W, 1.5), lin(W, f)
    return t


def make_engine(cfg: dict, tensors: dict, device: str, dtype=torch.float32, block_size=4, num_blocks=64, max_seqs=4, **kw):
    layers = ref_nekodra_modules if device == "cpu" else None
    model = NekodraForCausalLM(NekodraConfig.from_dict(cfg), layers=layers, dtype=dtype, device=device)
    model.load_tensors(tensors)
    return LLMEngine(model, model.config, block_size=block_size, num_kvcache_blocks=num_blocks, device=device,
                     max_num_seqs=max_seqs, dtype=dtype, **kw)


def oracle_logits(cfg: dict, tensors: dict, tokens, dtype=torch.float32):
    return ref_nekodra.forward(cfg, tensors, tokens, dtype)[0]


def per_position(got, want):
    """Per position: rms over the vocabulary of the difference with its mean removed, over the rms of the logits."""
    d = got.float() - want.float()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.float().pow(2).mean().sqrt()


def assert_close_to_oracle(got, cfg, ck, prompt, dtype, what="", f32_bound=5e-5):
    """float32: every position.  bfloat16: against what the oracle's own bfloat16 evaluation loses per position; a fault
    moves most positions, while rounding can turn a close call of a router (two experts whose scores differ by less
    than the rounding) and move that position and later ones that read it: at most one position in ten may exceed three
    times the oracle's loss, and the median must not move."""
    want = oracle_logits(cfg, ck, prompt, torch.float32)
    assert got.shape == want.shape
    err = per_position(got, want)
    if dtype == torch.float32:
        assert err.max().item() < f32_bound, (what, err.max().item(), int(err.argmax()))
        return
    noise = per_position(oracle_logits(cfg, ck, prompt, torch.bfloat16), want)
    limit = 3 * torch.clamp(noise, min=noise.median().item()) + 1e-3
    over = (err > limit).nonzero().flatten().tolist()
    assert len(over) <= max(1, err.numel() // 10), (what, (err / limit).topk(min(5, err.numel())).values.tolist())
    assert err.median().item() <= 2 * noise.median().item() + 1e-3, (what, err.median().item(), noise.median().item())


def layer_namespace(device: str):
    """The layer classes the model would use on this device: eager stand-ins on the CPU, HIP-backed on the GPU."""
    if device == "cpu":
        return ref_nekodra_modules
    from nanovllm_amd.model.nekodra import _default_layers
    return _default_layers()
