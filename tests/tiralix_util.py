"""Helpers of the Tiralix tests: small configurations, random checkpoints in the design's tensor names, and engines on
the CPU stand-ins or on the HIP layers.  The replay driver and the error measure are the Buvalix tests'."""
import math

import torch

import nanovllm_amd  # noqa: F401
from buvalix_util import paged_context, rel_err, replay  # noqa: F401
from nanovllm_amd.engine.llm_engine import LLMEngine
from nanovllm_amd.model.tiralix import TiralixConfig, TiralixForCausalLM
from oracle import ref_tiralix, ref_tiralix_modules


def dense(ff=44, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def mamba_layer(inner=40, state=6, dt_rank=5, conv=3, mlp="default"):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv},
            "mlp": dense() if mlp == "default" else mlp}


def parallel_layer(heads=6, kv_heads=3, dim=12, vdim=10, rot_dims=8, base=70.0, scaling="default", scale=None, rheads=2, rdim=9,
                   rvdim=14, decay=None, left_scale=0.8, right_scale=1.3, mlp="default"):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or 1.4 / math.sqrt(dim)}
    if rot_dims:
        left["rot"] = {"dims": rot_dims, "base": base}
        if scaling == "default":
            scaling = {"factor": 5.0, "original": 60, "fast": 6.0, "slow": 0.8}
        if scaling:
            left["rot"]["scaling"] = scaling
    decay = decay or [1.0 - 2.0 ** (-1.0 - 2.5 * h) for h in range(rheads)]
    return {"type": "parallel", "mlp": dense(28, 0.7) if mlp == "default" else mlp,
            "mixer": {"left": left, "right": {"heads": rheads, "dim": rdim, "vdim": rvdim, "decay": decay},
                      "left_scale": left_scale, "right_scale": right_scale}}


def config(layers, vocab=91, width=36, eps=1e-5, logit_scale=0.6, logit_softcap=12.0):
    return {"architecture": "Tiralix", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width,
            "logit_scale": logit_scale, "logit_softcap": logit_softcap}


def mamba_tensors(g, m, W, rn, lin, p=""):
    I, N, R = m["inner"], m["state"], m["dt_rank"]
    return {p + "in": lin(2 * I, W, 1.2), p + "conv": rn(I, m["conv"], std=0.6), p + "conv.b": rn(I, std=0.2),
            p + "x": lin(R + 2 * N, I, 2.0), p + "dt": lin(I, R), p + "dt.b": rn(I, std=1.0, mean=-3.0),
            p + "A_log": rn(I, N, std=0.7, mean=0.3), p + "D": rn(I, std=0.4, mean=0.8), p + "o": lin(W, I)}


def parallel_tensors(g, m, W, rn, lin, p=""):
    a, r = m["left"], m["right"]
    H, G, D, Dv, RH, RD, RV = a["heads"], a["kv_heads"], a["dim"], a["vdim"], r["heads"], r["dim"], r["vdim"]
    q, s = p + "left.", p + "right."
    return {q + "q": lin(H * D, W, 2.0), q + "k": lin(G * D, W, 2.0), q + "v": lin(G * Dv, W), q + "g": lin(H, W),
            q + "q.norm": rn(H * D, std=0.3, mean=1.3), q + "k.norm": rn(G * D, std=0.3, mean=1.3), q + "o": lin(W, H * Dv),
            s + "q": lin(RH * RD, W, 1.5), s + "k": lin(RH * RD, W, 1.5), s + "v": lin(RH * RV, W, 1.5), s + "g": lin(RH * RV, W),
            s + "norm": rn(RH * RV, std=0.2, mean=1.0), s + "o": lin(W, RH * RV)}


def random_checkpoint(cfg: dict, seed: int, dtype=torch.bfloat16) -> dict:
    """Tensors by checkpoint name, stored in bfloat16 like a file (so every dtype sees the same values)."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    rn = lambda *s, std=1.0, mean=0.0: (torch.randn(*s, generator=g) * std + mean).to(dtype)
    lin = lambda o, i, gain=1.0: rn(o, i, std=gain / math.sqrt(i))
    t = {"embed": rn(V, W), "final.norm": rn(W, std=0.2, mean=1.0)}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        t[p + "norm1"], t[p + "ls1"] = rn(W, std=0.2, mean=1.0), rn(W, std=0.3, mean=0.7)
        make = mamba_tensors if L["type"] == "mamba1" else parallel_tensors
        t.update(make(g, L["mixer"], W, rn, lin, p + "mix."))
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            t[p + "norm2"], t[p + "ls2"] = rn(W, std=0.2, mean=1.0), rn(W, std=0.3, mean=0.7)
            t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"] = lin(ff, W, 1.5), lin(ff, W, 1.5), lin(W, ff)
    return t


def make_engine(cfg: dict, tensors: dict, device: str, dtype=torch.float32, block_size=4, num_blocks=64, max_seqs=4, **kw):
    layers = ref_tiralix_modules if device == "cpu" else None
    model = TiralixForCausalLM(TiralixConfig.from_dict(cfg), layers=layers, dtype=dtype, device=device)
    model.load_tensors(tensors)
    return LLMEngine(model, model.config, block_size=block_size, num_kvcache_blocks=num_blocks, device=device,
                     max_num_seqs=max_seqs, dtype=dtype, **kw)


def oracle_logits(cfg: dict, tensors: dict, tokens, dtype=torch.float32):
    return ref_tiralix.forward(cfg, tensors, tokens, dtype)[0]


def layer_namespace(device: str):
    """The layer classes the model would use on this device: eager stand-ins on the CPU, HIP-backed on the GPU."""
    if device == "cpu":
        return ref_tiralix_modules
    from nanovllm_amd.model.tiralix import _default_layers
    return _default_layers()
