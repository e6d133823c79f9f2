"""Divadra: a decoder with a float32 residual stream that starts from a token embedding plus a hashed bigram embedding,
two RMS norms per layer (one per sublayer, both of the same stream), a short causal convolution in front of every
sublayer, two kinds of mixer chosen per layer, and a dense or table-routed feed-forward.

  * `mamba2`        a state-space layer: one in-projection cut into [z | x | B | C | dt]; x, B, C through a short causal
                    convolution with bias and SiLU; per head a state S [state, vdim] with a scalar decay per step,
                    S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x; the gate silu(z) comes before the grouped RMS
                    norm;
  * `parallel`      two mixers side by side on the same input, their outputs RMS-normed over the width and averaged:
                    left   grouped-query attention with q / k RMS-normed over the whole projection, rotate-half rotary,
                           values rotated by their position (and the sum turned back by the query's), sigmoid weights
                           with a per-head bias instead of a softmax, and visibility limited to fixed chunks of positions;
                    right  RWKV-style time mixing: every projection reads its own blend of the current and the previous
                           input, a low-rank data-dependent decay per key channel, a memory of decayed outer products read
                           with a bonus for the current token, per-head normalisation and a SiLU gate;
  * feed-forward    `dense`: down(relu(up h)^2);  `moe`: a table gives every token id its `top` experts, each
                    down(silu(gate h) * (up h)) with weight 1 / top;  absent where the config says null.

Per layer:  a = norm1(x), b = norm2(x);  x += mixer(a + conv1(a)) + ff(b + conv2(b)).

Per sequence the engine's state slots carry: the previous token id (bigram hash), the last taps - 1 norm outputs of
every layer (both sublayers' convolutions in one tensor), and per mixer the recurrent state and its carried inputs; the
attention caches rotated keys and rotated values in the engine's paged KV cache.

Every size and constant comes from config.json (`DivadraConfig.from_dict`).  The model is built from the package's
layers (`layers=` swaps in stand-ins, as for the other models); the matrix products are torch's.  What the design keeps
in 32 bits is kept there also when the model runs in bfloat16: the residual stream, norms, rotary angles, scores and
weights, both recurrences with their decays, step sizes and gates.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..engine.cache_spec import PagedKVSpec, SlotStateSpec
from ..utils.cache_context import get_context
from .buvalix import _FusedInputs, _linear


# ------------------------------------------------------------------------------------------------ configuration
@dataclass
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int                  # 0: plain causal
    rot_dims: int
    rot_base: float


@dataclass
class TimeMixConfig:
    heads: int
    dim: int


@dataclass
class StateSpaceConfig:
    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    conv: int


@dataclass
class FeedForwardConfig:
    kind: str                   # "dense" | "moe"
    ff: int
    experts: int = 0
    top: int = 0


@dataclass
class DivadraLayerConfig:
    kind: str                   # "mamba2" | "parallel"
    mixer: object               # StateSpaceConfig | (ChunkAttentionConfig, TimeMixConfig)
    mlp: FeedForwardConfig | None


@dataclass
class DivadraConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    canon_taps: int             # 0: no input convolution
    bigram_buckets: int         # 0: no bigram table
    bigram_mul_prev: int
    bigram_mul_cur: int
    layers: list = field(default_factory=list)
    eos_token_id: int | None = None
    max_position_embeddings: int | None = None      # the design has no position table: no bound

    @classmethod
    def from_dict(cls, d: dict) -> "DivadraConfig":
        layers = []
        for L in d["layers"]:
            m, kind = L["mixer"], L["type"]
            if kind == "mamba2":
                mc = StateSpaceConfig(heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]),
                                      groups=int(m.get("groups", 1)), norm_groups=int(m.get("norm_groups", 1)),
                                      conv=int(m["conv"]))
                if mc.heads % mc.groups or (mc.heads * mc.vdim) % mc.norm_groups or mc.conv < 1:
                    raise ValueError("mamba2: groups must divide heads, norm_groups the inner size, conv >= 1")
            elif kind == "parallel":
                a, r = m["left"], m["right"]
                rot = a.get("rot") or {}
                left = ChunkAttentionConfig(heads=int(a["heads"]), kv_heads=int(a["kv_heads"]), dim=int(a["dim"]),
                                            vdim=int(a["vdim"]), scale=float(a["scale"]),
                                            chunk=int((a.get("mask") or {}).get("size", 0)),
                                            rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)))
                if left.heads % left.kv_heads or left.rot_dims % 2 or left.rot_dims > left.dim or left.vdim % 2:
                    raise ValueError("parallel.left: kv_heads must divide heads; rot.dims even and at most dim; vdim even")
                mc = (left, TimeMixConfig(heads=int(r["heads"]), dim=int(r["dim"])))
            else:
                raise ValueError(f"unknown layer type {kind!r}")
            mlp = L.get("mlp")
            if mlp is not None:
                if mlp.get("kind") == "dense":
                    mlp = FeedForwardConfig("dense", int(mlp["ff"]))
                elif mlp.get("kind") == "moe":
                    mlp = FeedForwardConfig("moe", int(mlp["expert"]["ff"]), int(mlp["router"]["experts"]),
                                            int(mlp["router"]["top"]))
                    if not 1 <= mlp.top <= mlp.experts:
                        raise ValueError("router.top must lie in 1 .. router.experts")
                else:
                    raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
            layers.append(DivadraLayerConfig(kind, mc, mlp))
        bg = (d.get("embedding") or {}).get("bigram") or {}
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   canon_taps=int((d.get("canon") or {}).get("taps", 0)), bigram_buckets=int(bg.get("buckets", 0)),
                   bigram_mul_prev=int(bg.get("mul_prev", 0)), bigram_mul_cur=int(bg.get("mul_cur", 0)), layers=layers,
                   eos_token_id=d.get("eos_token_id"))


def _default_layers():
    from ..layers import chunk_attention, linear_memory, moe, parallel_stream, stream

    class _L:
        HashedBigramEmbedding = parallel_stream.HashedBigramEmbedding
        stream_boundary_pair = staticmethod(parallel_stream.stream_boundary_pair)
        ReluSquared = parallel_stream.ReluSquared
        CausalConvAdd = stream.CausalConvAdd
        ChunkSigmoidAttention = chunk_attention.ChunkSigmoidAttention
        TokenShiftMix = linear_memory.TokenShiftMix
        DecayMemory = linear_memory.DecayMemory
        ConvBiasSilu = linear_memory.ConvBiasSilu
        StateSpaceScan = linear_memory.StateSpaceScan
        group_rms_norm = staticmethod(linear_memory.group_rms_norm)
        TableExperts = moe.TableExperts
    return _L


# ------------------------------------------------------------------------------------------------ modules
class DivadraStateSpace(nn.Module):
    def __init__(self, m: StateSpaceConfig, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.m, self.eps, self._L = m, eps, L
        self.inner = m.heads * m.vdim
        self.conv_channels = self.inner + 2 * m.groups * m.state
        self.inp = _linear(width, self.inner + self.conv_channels + m.heads, False, dtype, device)
        self.conv = L.ConvBiasSilu(self.conv_channels, m.conv, device=device)
        self.scan = L.StateSpaceScan(m.heads, m.groups, m.state, m.vdim, device=device)
        self.norm = nn.Parameter(torch.ones(self.inner, dtype=torch.float32, device=device))
        self.o = _linear(self.inner, width, False, dtype, device)

    def cache_specs(self):
        m = self.m
        return [SlotStateSpec({"conv": ((m.conv - 1, self.conv_channels), None),
                               "state": ((m.heads, m.state, m.vdim), torch.float32)})]

    def names(self, p, t):
        return {p + "in": t + "inp.weight", p + "conv": t + "conv.weight", p + "conv.b": t + "conv.bias",
                p + "dt_bias": t + "scan.dt_bias", p + "A_log": t + "scan.A_log", p + "D": t + "scan.D",
                p + "norm": t + "norm", p + "o": t + "o.weight"}

    def finalize(self):
        pass

    def forward(self, h, positions, caches):
        m, inner = self.m, self.inner
        cache = caches[0]
        proj = self.inp(h)
        z, xbc, dt_raw = proj[:, :inner], proj[:, inner:inner + self.conv_channels], proj[:, inner + self.conv_channels:]
        xbc = self.conv(xbc, cache["conv"])
        gn = m.groups * m.state
        x = xbc[:, :inner].unflatten(1, (m.heads, m.vdim))
        B = xbc[:, inner:inner + gn].unflatten(1, (m.groups, m.state))
        C = xbc[:, inner + gn:].unflatten(1, (m.groups, m.state))
        y = self.scan(x, B, C, dt_raw, z, cache["state"])
        return [self.o(self._L.group_rms_norm(y, self.norm, m.norm_groups, self.eps, h.dtype))], []


class DivadraChunkAttention(nn.Module, _FusedInputs):
    _inputs = ("q", "k", "v")

    def __init__(self, m: ChunkAttentionConfig, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.m = m
        self.q = _linear(width, m.heads * m.dim, False, dtype, device)
        self.k = _linear(width, m.kv_heads * m.dim, False, dtype, device)
        self.v = _linear(width, m.kv_heads * m.vdim, False, dtype, device)
        self.o = _linear(m.heads * m.vdim, width, False, dtype, device)
        self.attn = L.ChunkSigmoidAttention(m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.chunk, m.rot_dims, m.rot_base,
                                            eps, device=device)

    def cache_spec(self):
        return PagedKVSpec(self.m.kv_heads, self.m.dim, self.m.vdim)

    def names(self, p, t):
        n = {p + x: t + x + ".weight" for x in ("q", "k", "v", "o")}
        n.update({p + "q.norm": t + "attn.q_norm", p + "k.norm": t + "attn.k_norm", p + "pb": t + "attn.head_bias"})
        return n

    def finalize(self):
        self._fuse(self._inputs)

    def forward(self, h, positions, cache):
        m = self.m
        q, k, v = self._project(h, self._inputs)
        o = self.attn(q.unflatten(1, (m.heads, m.dim)), k.unflatten(1, (m.kv_heads, m.dim)),
                      v.unflatten(1, (m.kv_heads, m.vdim)), positions, cache[0], cache[1])
        return self.o(o)


class DivadraTimeMix(nn.Module):
    _mixes = ("r", "k", "v", "g", "w")

    def __init__(self, m: TimeMixConfig, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.m, self.width = m, width
        n = m.heads * m.dim
        for name in ("r", "k", "v", "g"):
            setattr(self, name, _linear(width, n, False, dtype, device))
        # the low-rank width is the file's (w1: [rank, width]); 1 here, resized when the weights arrive
        self.w1 = _linear(width, 1, False, dtype, device)
        self.w2 = _linear(1, n, False, dtype, device)
        self.o = _linear(n, width, False, dtype, device)
        self.shift = L.TokenShiftMix(len(self._mixes), width, device=device)
        self.memory = L.DecayMemory(m.heads, m.dim, m.dim, eps, device=device)
        self._stacked = None

    def cache_spec(self):
        m = self.m
        return SlotStateSpec({"prev": ((self.width,), None), "state": ((m.heads, m.dim, m.dim), torch.float32)})

    def names(self, p, t):
        n = {p + x: t + x + ".weight" for x in ("r", "k", "v", "g", "w1", "w2", "o")}
        n.update({p + "w0": t + "memory.w_bias", p + "u": t + "memory.bonus", p + "norm": t + "memory.norm_weight"})
        return n

    def finalize(self):
        if self.w2.weight.shape[1] != self.w1.weight.shape[0]:
            raise ValueError("low-rank decay projections do not chain")
        # r, k, v, g read different blends: one batched product over the stacked weights (the Linear weights become views)
        # (stored transposed: a bfloat16 batched product takes a contiguous right operand only, a transposed view can fault
        # the GPU)
        w = torch.stack([getattr(self, n).weight.data.t() for n in ("r", "k", "v", "g")])
        for i, n in enumerate(("r", "k", "v", "g")):
            getattr(self, n).weight.data = w[i].t()
        self._stacked = w

    def forward(self, h, positions, cache):
        H, D = self.m.heads, self.m.dim
        mixes = self.shift(h, cache["prev"])                                      # [5, T, W]
        w = self._stacked
        if w is not None and w.device == h.device and w.dtype == h.dtype:
            r, k, v, g = torch.bmm(mixes[:4], w).unbind(0)
        else:
            r, k, v, g = (getattr(self, n)(mixes[i]) for i, n in enumerate(("r", "k", "v", "g")))
        w_raw = self.w2(torch.tanh(self.w1(mixes[4]).float()).to(h.dtype))
        o = self.memory(r.unflatten(1, (H, D)), k.unflatten(1, (H, D)), v.unflatten(1, (H, D)), w_raw, g, cache["state"])
        return self.o(o)


class DivadraParallelMixer(nn.Module):
    def __init__(self, m, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.left = DivadraChunkAttention(m[0], width, eps, L, dtype, device)
        self.right = DivadraTimeMix(m[1], width, eps, L, dtype, device)
        self.left_out = nn.Parameter(torch.ones(width, dtype=torch.float32, device=device))
        self.right_out = nn.Parameter(torch.ones(width, dtype=torch.float32, device=device))

    def cache_specs(self):
        return [self.left.cache_spec(), self.right.cache_spec()]

    def names(self, p, t):
        n = {p + "left.out": t + "left_out", p + "right.out": t + "right_out"}
        n.update(self.left.names(p + "left.", t + "left."))
        n.update(self.right.names(p + "right.", t + "right."))
        return n

    def finalize(self):
        self.left.finalize()
        self.right.finalize()

    def forward(self, h, positions, caches):
        """Returns (outputs added as they are, outputs that are RMS-normed with their weight and averaged)."""
        return [], [(self.left(h, positions, caches[0]), self.left_out), (self.right(h, positions, caches[1]), self.right_out)]


class DivadraDenseFF(nn.Module):
    def __init__(self, c: FeedForwardConfig, width: int, L, dtype, device):
        super().__init__()
        self.up = _linear(width, c.ff, False, dtype, device)
        self.down = _linear(c.ff, width, False, dtype, device)
        self.act = L.ReluSquared()

    def forward(self, h, token_ids):
        """Returns (output in the matmul dtype or None, float32 parts [T, n, W] or None, weight of the parts)."""
        return self.down(self.act(self.up(h))), None, 1.0


class DivadraTableMoE(nn.Module):
    def __init__(self, c: FeedForwardConfig, vocab: int, width: int, L, dtype, device):
        super().__init__()
        self.c = c
        self.register_buffer("table", torch.zeros(vocab, c.top, dtype=torch.int32, device=device))
        # per expert [gate rows | up rows] x width, and down [width, ff]
        self.gate_up = nn.Parameter(torch.zeros(c.experts, 2 * c.ff, width, dtype=dtype, device=device))
        self.down = nn.Parameter(torch.zeros(c.experts, width, c.ff, dtype=dtype, device=device))
        self.experts = L.TableExperts(c.top)

    def forward(self, h, token_ids):
        return None, self.experts(h, self.table, token_ids, self.gate_up, self.down), 1.0 / self.c.top


class DivadraLayer(nn.Module):
    def __init__(self, lc: DivadraLayerConfig, cfg: DivadraConfig, L, dtype, device):
        super().__init__()
        W, eps = cfg.hidden_size, cfg.norm_eps
        self.norm1 = nn.Parameter(torch.ones(W, dtype=torch.float32, device=device))
        self.norm2 = nn.Parameter(torch.ones(W, dtype=torch.float32, device=device)) if lc.mlp is not None else None
        self.n_inputs = 2 if lc.mlp is not None else 1
        # both sublayers' input convolutions as one over [norm1 output | norm2 output]
        self.canon = L.CausalConvAdd(W * self.n_inputs, cfg.canon_taps, device=device) if cfg.canon_taps else None
        if lc.kind == "mamba2":
            self.mix = DivadraStateSpace(lc.mixer, W, eps, L, dtype, device)
        else:
            self.mix = DivadraParallelMixer(lc.mixer, W, eps, L, dtype, device)
        if lc.mlp is None:
            self.mlp = None
        elif lc.mlp.kind == "dense":
            self.mlp = DivadraDenseFF(lc.mlp, W, L, dtype, device)
        else:
            self.mlp = DivadraTableMoE(lc.mlp, cfg.vocab_size, W, L, dtype, device)

    def norms(self):
        return [self.norm1] if self.norm2 is None else [self.norm1, self.norm2]


class DivadraForCausalLM(nn.Module):
    #: the in-tree library this model's layers need (`nanovllm_amd._lib.build(target)`)
    kernel_library = "mixers"
    #: a cached prompt prefix cannot be taken over: the carried state at its end is not kept
    prefix_caching = False

    def __init__(self, cfg: DivadraConfig, layers=None, dtype: torch.dtype = torch.bfloat16, device=None):
        super().__init__()
        L = layers if layers is not None else _default_layers()
        self.config, self.dtype, self._L = cfg, dtype, L
        self.embed = L.HashedBigramEmbedding(cfg.vocab_size, cfg.hidden_size, cfg.bigram_buckets, cfg.bigram_mul_prev,
                                             cfg.bigram_mul_cur, cfg.norm_eps, dtype=dtype, device=device)
        self.layers = nn.ModuleList(DivadraLayer(lc, cfg, L, dtype, device) for lc in cfg.layers)
        self.final_norm = nn.Parameter(torch.ones(cfg.hidden_size, dtype=torch.float32, device=device))
        self.head = _linear(cfg.hidden_size, cfg.vocab_size, False, dtype, device)
        self._caches = None

    # ---- weights ----------------------------------------------------------------------------------------
    def checkpoint_names(self) -> dict[str, str]:
        """checkpoint tensor name -> parameter name of this module tree (experts, tables and the paired input
        convolutions are placed separately)."""
        names = {"embed": "embed.weight", "embed.norm": "embed.norm", "head": "head.weight", "final.norm": "final_norm"}
        if self.embed.bigram is not None:
            names["bigram"] = "embed.bigram"
        for i, layer in enumerate(self.layers):
            p, t = f"l{i}.", f"layers.{i}."
            names[p + "norm1"] = t + "norm1"
            if layer.norm2 is not None:
                names[p + "norm2"] = t + "norm2"
            names.update(layer.mix.names(p + "mix.", t + "mix."))
            if isinstance(layer.mlp, DivadraDenseFF):
                names[p + "mlp.up"], names[p + "mlp.down"] = t + "mlp.up.weight", t + "mlp.down.weight"
        return names

    def load_tensors(self, tensors: dict[str, torch.Tensor]) -> None:
        """Copy checkpoint tensors (by checkpoint name) into the parameters.  The low-rank width of the decay projection
        is the file's; the experts of a layer are stacked into [experts, rows, cols] tensors, the blend weights of the time
        mixing into [blends, width]; the two input convolutions of a layer become one over both norm outputs."""
        names = self.checkpoint_names()
        params = dict(self.named_parameters())
        seen = set()

        def take(name):
            if name not in tensors:
                raise KeyError(f"checkpoint lacks {name}")
            seen.add(name)
            return tensors[name]

        with torch.no_grad():
            W = self.config.hidden_size
            for i, layer in enumerate(self.layers):
                p = f"l{i}."
                if layer.canon is not None:
                    for j in range(layer.n_inputs):
                        t = take(f"{p}canon{j + 1}")
                        if t.shape != (W, self.config.canon_taps):
                            raise ValueError(f"{p}canon{j + 1}: shape {tuple(t.shape)} does not match the configuration")
                        layer.canon.weight[j * W:(j + 1) * W].copy_(t)
                if isinstance(layer.mix, DivadraParallelMixer):
                    right = layer.mix.right
                    for j, n in enumerate(right._mixes):
                        t = take(f"{p}mix.right.mu.{n}")
                        if t.shape != (W,):
                            raise ValueError(f"{p}mix.right.mu.{n}: shape {tuple(t.shape)} does not match the width")
                        right.shift.mu[j].copy_(t)
                if isinstance(layer.mlp, DivadraTableMoE):
                    c = layer.mlp.c
                    table = take(p + "mlp.table")
                    if table.shape != layer.mlp.table.shape or int(table.min()) < 0 or int(table.max()) >= c.experts:
                        raise ValueError(f"{p}mlp.table does not match the configuration")
                    layer.mlp.table.copy_(table)
                    for e in range(c.experts):
                        q = f"{p}mlp.e{e}."
                        gu = torch.cat([take(q + "gate"), take(q + "up")], dim=0)
                        dn = take(q + "down")
                        if gu.shape != layer.mlp.gate_up.shape[1:] or dn.shape != layer.mlp.down.shape[1:]:
                            raise ValueError(f"{q}*: expert shapes do not match the configuration")
                        layer.mlp.gate_up[e].copy_(gu)
                        layer.mlp.down[e].copy_(dn)
            for ck, pn in names.items():
                t, prm = take(ck), params[pn]
                if t.shape != prm.shape:
                    free = pn.endswith((".w1.weight", ".w2.weight"))
                    if not free or t.dim() != prm.dim():
                        raise ValueError(f"{ck}: checkpoint shape {tuple(t.shape)} != parameter {tuple(prm.shape)}")
                    prm.data = torch.empty(t.shape, dtype=prm.dtype, device=prm.device)
                prm.copy_(t)
        extra = sorted(set(tensors) - seen)
        if extra:
            raise KeyError(f"checkpoint has tensors the model does not know, e.g. {extra[:3]}")
        self.finalize()

    def finalize(self) -> "DivadraForCausalLM":
        for layer in self.layers:
            layer.mix.finalize()
        return self

    # ---- caches -------------------------------------------------------------------------------------------
    def cache_specs(self) -> list:
        """The previous token id first; then per layer the convolutions' carried inputs (when the design has them) and
        the mixer's caches (a paged KV cache and / or state slots)."""
        cfg = self.config
        specs = [SlotStateSpec({"token": ((), torch.int64)})]
        for layer in self.layers:
            if layer.canon is not None:
                specs.append(SlotStateSpec({"inputs": ((cfg.canon_taps - 1, cfg.hidden_size * layer.n_inputs), torch.float32)}))
            specs.extend(layer.mix.cache_specs())
        return specs

    def bind_caches(self, caches: list) -> None:
        self._prev_token = caches[0]["token"]
        at, bound = 1, []
        for layer in self.layers:
            conv = None
            if layer.canon is not None:
                conv = caches[at]["inputs"]
                at += 1
            n = len(layer.mix.cache_specs())
            bound.append((conv, caches[at:at + n]))
            at += n
        assert at == len(caches)
        self._caches = bound

    # ---- forward ------------------------------------------------------------------------------------------
    def forward(self, input_ids, positions, logits_rows=None, streams: list | None = None):
        """Returns float32 logits [T or len(logits_rows), vocab].  streams: a list that receives the residual stream
        after every layer."""
        if self._caches is None:
            raise RuntimeError("caches are not bound: the model runs through the engine's cache and state manager")
        cfg, L, dt = self.config, self._L, self.dtype
        eps, W = cfg.norm_eps, cfg.hidden_size
        ctx = get_context()
        x = self.embed(input_ids, positions, self._prev_token)
        h32, _ = L.stream_boundary_pair(x, norms=self.layers[0].norms(), eps=eps)
        last = len(self.layers) - 1
        h = None
        for i, layer in enumerate(self.layers):
            ctx.layer_idx = i
            conv_state, caches = self._caches[i]
            hc = layer.canon(h32, conv_state, dt) if layer.canon is not None else h32.to(dt)
            adds, normed = layer.mix(hc[:, :W], positions, caches)
            parts, scale = None, 1.0
            if layer.mlp is not None:
                y, parts, scale = layer.mlp(hc[:, W:], input_ids)
                if y is not None:
                    adds = adds + [y]
            if i == last and logits_rows is not None and streams is None:
                # only the asked rows go on: the caches and states of this step are complete
                x = x[logits_rows]
                adds = [a[logits_rows] for a in adds]
                normed = [(n[logits_rows], w) for n, w in normed]
                parts = parts[logits_rows] if parts is not None else None
                logits_rows = None
            nxt = self.layers[i + 1].norms() if i < last else [self.final_norm]
            kw = dict(adds=adds, parts=parts, parts_scale=scale, normed=normed, normed_mult=0.5, eps=eps)
            if streams is not None:
                L.stream_boundary_pair(x, **kw)
                streams.append(x.clone())
                kw = dict(eps=eps)
            h32, h = L.stream_boundary_pair(x, norms=nxt, out_dtype=dt if i == last else None, want_f32=i < last, **kw)
        if logits_rows is not None:
            h = h[logits_rows]
        return self.head(h).float()
