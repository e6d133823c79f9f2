"""Nekodra: a decoder with a float32 residual stream that starts from a token embedding plus a learned position vector
and that every layer reads through TWO layer norms with biases, one per parallel sublayer:

    x += mixer(norm1(x)) + ff(norm2(x))

  * mixer         latent attention without positions: q = W_q h; keys and values are per-head projections of one RMS-normed
                  low-rank latent per token; a learned sink joins every head's softmax denominator; the heads' outputs are
                  multiplied by sigmoid(W_g h) in front of the output projection.  A layer may read the latents of an
                  earlier layer (`kv_from`) with its own queries and up-projections, and then has none of its own;
  * feed-forward  SiLU-gated experts chosen by softmax scores plus a correction, weighted by the plain scores times a
                  constant; the last ones scored are identity experts that hand their input through; plus a shared expert
                  that runs for every token; absent where the config says null.

Only the latent is cached, one paged row per token and layer that has its own: attention runs in latent space (the key
up-projection is applied to the query, the value up-projection to the attention output), i.e. as multi-query attention with
one key "head" of kv_rank columns whose key and value are the same row.  A layer with `kv_from` is bound to the cache of
the layer it names.  There is no other per-sequence state, so cached prompt prefixes are shared as for the
uniform-layer models.

Every size and constant comes from config.json (`NekodraConfig.from_dict`).  The model is built from the package's layers
(`layers=` swaps in stand-ins, as for the other models); the plain matrix products are torch's.  What the design keeps in 32
bits is kept there also when the model runs in bfloat16: the residual stream, norms, attention scores and weights,
router logits, scores and weights, and the sum of the experts' outputs.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..engine.cache_spec import PagedKVSpec
from ..utils.cache_context import get_context
from .buvalix import _FusedInputs, _linear


# ------------------------------------------------------------------------------------------------ configuration
@dataclass
class LatentMixerConfig:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    kv_from: int | None         # the layer whose latents are read; None: its own


@dataclass
class RoutedFFConfig:
    experts: int                # experts with tensors
    identity: int               # experts without, scored behind them
    top: int
    scale: float
    ff: int
    shared_ff: int              # 0: no shared expert


@dataclass
class NekodraLayerConfig:
    mixer: LatentMixerConfig
    mlp: RoutedFFConfig | None


@dataclass
class NekodraConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    max_position_embeddings: int
    layers: list = field(default_factory=list)
    eos_token_id: int | None = None

    @classmethod
    def from_dict(cls, d: dict) -> "NekodraConfig":
        layers = []
        for i, L in enumerate(d["layers"]):
            if L["type"] != "latent_attention":
                raise ValueError(f"unknown layer type {L['type']!r}")
            m = L["mixer"]
            src = m.get("kv_from")
            mc = LatentMixerConfig(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
                                   scale=float(m["scale"]), kv_from=None if src is None else int(src))
            if src is not None:
                j = mc.kv_from
                if not 0 <= j < i or layers[j].mixer.kv_from is not None or layers[j].mixer.kv_rank != mc.kv_rank:
                    raise ValueError(f"layer {i}: kv_from must name an earlier layer with latents of its own and the same kv_rank")
            mlp = L.get("mlp")
            if mlp is not None:
                if mlp.get("kind") != "moe":
                    raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
                r = mlp["router"]
                mlp = RoutedFFConfig(experts=int(r["experts"]), identity=int(r.get("identity") or 0), top=int(r["top"]),
                                     scale=float(r.get("scale", 1.0)), ff=int(mlp["expert"]["ff"]),
                                     shared_ff=int((mlp.get("shared") or {}).get("ff", 0)))
                if mlp.experts < 1 or mlp.identity < 0 or not 1 <= mlp.top <= mlp.experts + mlp.identity:
                    raise ValueError("router.top must lie in 1 .. experts + identity, with at least one expert")
            layers.append(NekodraLayerConfig(mc, mlp))
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   max_position_embeddings=int(d["max_positions"]), layers=layers, eos_token_id=d.get("eos_token_id"))


def _default_layers():
    from ..layers import activation, latent_attention, layernorm, moe, parallel_stream

    class _L:
        PositionEmbedding = parallel_stream.PositionEmbedding
        layernorm_pair_boundary = staticmethod(parallel_stream.layernorm_pair_boundary)
        LayerNorm = layernorm.LayerNorm
        UnrotatedLatentAttention = latent_attention.UnrotatedLatentAttention
        HeadLinear = latent_attention.HeadLinear
        SoftmaxRouter = moe.SoftmaxRouter
        SiluExperts = moe.SiluExperts
        SiluAndMulRows = activation.SiluAndMulRows
    return _L


# ------------------------------------------------------------------------------------------------ modules
class NekodraAttention(nn.Module, _FusedInputs):
    def __init__(self, m: LatentMixerConfig, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.m = m
        H = m.heads
        self.q = _linear(width, H * m.dim, False, dtype, device)
        self.g = _linear(width, H * m.vdim, False, dtype, device)
        self._inputs = ("q", "g")
        if m.kv_from is None:
            self.dkv = _linear(width, m.kv_rank, False, dtype, device)
            self._inputs += ("dkv",)
        # the key up-projection acts on the query (stored transposed per head, [H, rank, dim]), the value up-projection on
        # the attention output ([H, vdim, rank], as in the checkpoint)
        self.uk = L.HeadLinear(H, m.dim, m.kv_rank, dtype=dtype, device=device)
        self.uv = L.HeadLinear(H, m.kv_rank, m.vdim, dtype=dtype, device=device)
        self.o = _linear(H * m.vdim, width, False, dtype, device)
        self.attn = L.UnrotatedLatentAttention(H, m.kv_rank, m.scale, eps, own_latent=m.kv_from is None, use_sink=True, device=device)

    def names(self, p, t):
        n = {p + x: t + x + ".weight" for x in self._inputs + ("o",)}
        n[p + "sink"] = t + "attn.sink"
        if self.m.kv_from is None:
            n[p + "dkv.norm"] = t + "attn.latent_norm"
        return n

    def place(self, p, take):
        m = self.m
        for name, rows in (("uk", m.dim), ("uv", m.vdim)):
            t = take(p + name)
            if t.shape != (m.heads * rows, m.kv_rank):
                raise ValueError(f"{p}{name}: shape {tuple(t.shape)} does not match the configuration")
            t = t.reshape(m.heads, rows, m.kv_rank)
            getattr(self, name).weight.copy_(t.transpose(1, 2) if name == "uk" else t)

    def finalize(self):
        self._fuse(self._inputs)

    def forward(self, h, cache):
        rows = self._project(h, self._inputs)
        q_lat = self.uk(rows[0])
        o_lat = self.attn(q_lat, rows[2] if self.m.kv_from is None else None, cache[0], cache[1])
        return self.o(self.uv(o_lat, rows[1]))


class NekodraMoE(nn.Module):
    def __init__(self, c: RoutedFFConfig, width: int, L, dtype, device):
        super().__init__()
        self.c = c
        self.router_weight = nn.Parameter(torch.zeros(c.experts + c.identity, width, dtype=torch.float32, device=device))
        self.router = L.SoftmaxRouter(c.experts + c.identity, c.top, c.scale, device=device)
        # per expert [gate rows | up rows] x width, and down [width, ff]
        self.gate_up = nn.Parameter(torch.zeros(c.experts, 2 * c.ff, width, dtype=dtype, device=device))
        self.down = nn.Parameter(torch.zeros(c.experts, width, c.ff, dtype=dtype, device=device))
        self.experts = L.SiluExperts()
        if c.shared_ff:
            self.shared_in = _linear(width, 2 * c.shared_ff, False, dtype, device)      # gate rows, then up rows
            self.shared_down = _linear(c.shared_ff, width, False, dtype, device)
            self.shared_act = L.SiluAndMulRows()

    def place(self, p, take, has):
        c, W = self.c, self.router_weight.shape[1]
        if has(p + "correction"):
            if self.router.correction is None:
                self.router.correction = nn.Parameter(torch.zeros(c.experts + c.identity, dtype=torch.float32,
                                                                  device=self.router_weight.device))
            self.router.correction.copy_(take(p + "correction").reshape(-1))
        else:
            self.router.correction = None

        def unit(q, gate_up, down, ff):
            g, u, d = take(q + "gate"), take(q + "up"), take(q + "down")
            if g.shape != (ff, W) or u.shape != (ff, W) or d.shape != (W, ff):
                raise ValueError(f"{q}*: shapes do not match the configuration")
            gate_up[:ff].copy_(g)
            gate_up[ff:].copy_(u)
            down.copy_(d)
        for e in range(c.experts):
            unit(f"{p}e{e}.", self.gate_up[e], self.down[e], c.ff)
        if c.shared_ff:
            unit(p + "shared.", self.shared_in.weight, self.shared_down.weight, c.shared_ff)

    def forward(self, h, h32):
        """Returns the keyword arguments of the stream boundary: the shared expert's output (or none) and the routed part."""
        ids, weights = self.router(F.linear(h32 if h32 is not None else h, self.router_weight))
        routed = (self.experts(h, ids, weights, self.gate_up, self.down), ids, weights, self.c.experts, h)
        shared = [self.shared_down(self.shared_act(self.shared_in(h)))] if self.c.shared_ff else []
        return shared, routed


class NekodraLayer(nn.Module):
    def __init__(self, lc: NekodraLayerConfig, cfg: NekodraConfig, L, dtype, device):
        super().__init__()
        W, eps = cfg.hidden_size, cfg.norm_eps
        self.norm1 = L.LayerNorm(W, eps, device=device)
        self.mix = NekodraAttention(lc.mixer, W, eps, L, dtype, device)
        self.norm2 = L.LayerNorm(W, eps, device=device) if lc.mlp is not None else None
        self.mlp = NekodraMoE(lc.mlp, W, L, dtype, device) if lc.mlp is not None else None


class NekodraForCausalLM(nn.Module):
    #: the in-tree library this model's layers need (`nanovllm_amd._lib.build(target)`)
    kernel_library = "mixers"
    #: everything a sequence leaves behind is in its pages: a cached prompt prefix can be taken over
    prefix_caching = True

    def __init__(self, cfg: NekodraConfig, layers=None, dtype: torch.dtype = torch.bfloat16, device=None):
        super().__init__()
        L = layers if layers is not None else _default_layers()
        self.config, self.dtype, self._L = cfg, dtype, L
        self.embed = L.PositionEmbedding(cfg.vocab_size, cfg.max_position_embeddings, cfg.hidden_size, dtype=dtype, device=device)
        self.layers = nn.ModuleList(NekodraLayer(lc, cfg, L, dtype, device) for lc in cfg.layers)
        self.final_norm = L.LayerNorm(cfg.hidden_size, cfg.norm_eps, device=device)
        self.head = _linear(cfg.hidden_size, cfg.vocab_size, False, dtype, device)
        self._caches: list | None = None

    # ---- weights ----------------------------------------------------------------------------------------
    def checkpoint_names(self) -> dict[str, str]:
        """checkpoint tensor name -> parameter name of this module tree (up-projections, experts, the shared expert and the
        correction are placed separately)."""
        names = {"embed": "embed.weight", "pos": "embed.pos", "head": "head.weight", "final.norm": "final_norm.weight",
                 "final.norm.b": "final_norm.bias"}
        for i, layer in enumerate(self.layers):
            p, t = f"l{i}.", f"layers.{i}."
            for n in ("norm1", "norm2") if layer.mlp is not None else ("norm1",):
                names[p + n] = t + n + ".weight"
                names[p + n + ".b"] = t + n + ".bias"
            names.update(layer.mix.names(p + "mix.", t + "mix."))
            if layer.mlp is not None:
                names[p + "mlp.router"] = t + "mlp.router_weight"
        return names

    def load_tensors(self, tensors: dict[str, torch.Tensor]) -> None:
        """Copy checkpoint tensors (by checkpoint name) into the parameters.  The experts of a layer are stacked into
        [experts, rows, cols] tensors, the up-projections cut per head (the key one transposed)."""
        names = self.checkpoint_names()
        params = dict(self.named_parameters())
        seen = set()

        def take(name):
            if name not in tensors:
                raise KeyError(f"checkpoint lacks {name}")
            seen.add(name)
            return tensors[name]

        with torch.no_grad():
            for i, layer in enumerate(self.layers):
                layer.mix.place(f"l{i}.mix.", take)
                if layer.mlp is not None:
                    layer.mlp.place(f"l{i}.mlp.", take, tensors.__contains__)
                else:                                   # an unused second norm may come with the file
                    seen.update(n for n in (f"l{i}.norm2", f"l{i}.norm2.b") if n in tensors)
            for ck, pn in names.items():
                t, prm = take(ck), params[pn]
                if t.shape != prm.shape:
                    raise ValueError(f"{ck}: checkpoint shape {tuple(t.shape)} != parameter {tuple(prm.shape)}")
                prm.copy_(t)
        extra = sorted(set(tensors) - seen)
        if extra:
            raise KeyError(f"checkpoint has tensors the model does not know, e.g. {extra[:3]}")
        self.finalize()

    def finalize(self) -> "NekodraForCausalLM":
        for layer in self.layers:
            layer.mix.finalize()
        return self

    # ---- caches -------------------------------------------------------------------------------------------
    def cache_specs(self) -> list:
        """One paged latent cache per layer that has latents of its own: key and value are the same row."""
        return [PagedKVSpec(1, c.mixer.kv_rank, c.mixer.kv_rank, value_in_key=True)
                for c in self.config.layers if c.mixer.kv_from is None]

    def bind_caches(self, caches: list) -> None:
        own, bound = iter(caches), []
        for c in self.config.layers:
            bound.append(next(own) if c.mixer.kv_from is None else bound[c.mixer.kv_from])
        assert next(own, None) is None
        self._caches = bound

    # ---- forward ------------------------------------------------------------------------------------------
    def forward(self, input_ids, positions, logits_rows=None, streams: list | None = None):
        """Returns float32 logits [T or len(logits_rows), vocab].  streams: a list that receives the residual stream
        after every layer."""
        if self._caches is None:
            raise RuntimeError("caches are not bound: the model runs through the engine's cache and state manager")
        L, dt = self._L, self.dtype
        ctx = get_context()

        def boundary(x, norm1, layer=None, **kw):
            second = layer.norm2 if layer is not None else None
            # a router reads its norm in float32 (in a float32 model that is the norm itself)
            return L.layernorm_pair_boundary(x, norm_a=(norm1.weight, norm1.bias),
                                             norm_b=(second.weight, second.bias) if second is not None else None,
                                             eps=norm1.eps, out_dtype=dt, want_f32_b=second is not None and dt != torch.float32, **kw)

        x = self.embed(input_ids, positions)
        h1, h2, h2_32 = boundary(x, self.layers[0].norm1, self.layers[0])
        last = len(self.layers) - 1
        for i, layer in enumerate(self.layers):
            ctx.layer_idx = i
            y = layer.mix(h1, self._caches[i])
            if i == last and logits_rows is not None and streams is None:
                # behind the last mixer only the asked rows go on: the caches of this step are complete
                x, y = x[logits_rows], y[logits_rows]
                h2, h2_32 = (t[logits_rows] if t is not None else None for t in (h2, h2_32))
                logits_rows = None
            shared, routed = layer.mlp(h2, h2_32) if layer.mlp is not None else ([], None)
            if i < last:
                h1, h2, h2_32 = boundary(x, self.layers[i + 1].norm1, self.layers[i + 1], adds=[y] + shared, routed=routed)
            else:
                h1, _, _ = boundary(x, self.final_norm, adds=[y] + shared, routed=routed)
            if streams is not None:
                streams.append(x.clone())
        if logits_rows is not None:
            h1 = h1[logits_rows]
        return self.head(h1).float()
