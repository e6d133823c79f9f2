"""Tiralix: a decoder with a float32 residual stream that starts as the token embedding and that the sublayers read AS IT IS;
only their outputs are RMS-normed, scaled per column and added:

    x += ls1 * norm1(mixer(x));   x += ls2 * norm2(ff(x));   logits = cap * tanh(logit_scale * (embed final_norm(x)) / cap)

  * `mamba1`     a selective scan: [x | z] = W_in h, x through a short causal convolution with bias and SiLU,
                 [dt | B | C] = W_x x, dt = softplus(W_dt dt + b), per channel S <- exp(dt A) S + dt x B, y = S C + D x,
                 W_o (y * silu(z));
  * `parallel`   two mixers on the same input, left_scale * left + right_scale * right.  Left: grouped-query softmax attention;
                 q and k RMS-normed over their whole projection, rotate-half rotary with blended frequencies on the first
                 dimensions of every head, one sigmoid gate per head on the way out.  Right: linear attention with one fixed
                 decay per head on SiLU-activated q, k, v, its read-out RMS-normed over all heads and gated per column;
  * feed-forward `dense`: a gated unit with clamped branches;  absent where the config says null.

Per sequence the engine's state slots carry, per mixer, the recurrent state in float32 and (`mamba1`) the last inputs of the
convolution; the attention caches prepared keys and values in the engine's paged KV cache.

Every size and constant comes from config.json (`TiralixConfig.from_dict`).  The model is built from the package's layers
(`layers=` swaps in stand-ins, as for the other models); the matrix products are torch's: the input projections of a mixer
run as one product, and so do the two output projections of a parallel mixer (its constants are applied in front of it).
What the design keeps in 32 bits is kept there also when the model runs in bfloat16: the residual stream, norms, rotary
angles, scores and weights, and both recurrences with their decays, step sizes and exponentials.
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
class SelectiveScanConfig:
    inner: int
    state: int
    dt_rank: int
    conv: int                   # taps


@dataclass
class GatedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int               # 0: no rotary
    rot_base: float
    rot_scaling: dict | None    # factor, original, fast, slow


@dataclass
class LinearAttentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: list                 # one per head


@dataclass
class ParallelConfig:
    left: GatedAttentionConfig
    right: LinearAttentionConfig
    left_scale: float
    right_scale: float


@dataclass
class FeedForwardConfig:
    ff: int
    limit: float


@dataclass
class TiralixLayerConfig:
    kind: str                   # "mamba1" | "parallel"
    mixer: object
    mlp: FeedForwardConfig | None


@dataclass
class TiralixConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    logit_scale: float
    logit_softcap: float        # 0: none
    layers: list = field(default_factory=list)
    eos_token_id: int | None = None
    max_position_embeddings: int | None = None      # the design has no position table: no bound

    @classmethod
    def from_dict(cls, d: dict) -> "TiralixConfig":
        layers = []
        for L in d["layers"]:
            m, kind = L["mixer"], L["type"]
            if kind == "mamba1":
                mc = SelectiveScanConfig(int(m["inner"]), int(m["state"]), int(m["dt_rank"]), int(m["conv"]))
                if min(mc.inner, mc.state, mc.dt_rank, mc.conv) < 1:
                    raise ValueError("mamba1: sizes must be positive")
            elif kind == "parallel":
                a, r = m["left"], m["right"]
                rot = a.get("rot") or {}
                left = GatedAttentionConfig(int(a["heads"]), int(a.get("kv_heads", a["heads"])), int(a["dim"]), int(a["vdim"]),
                                            float(a["scale"]), int(rot.get("dims", 0)), float(rot.get("base", 10000.0)),
                                            rot.get("scaling") or None)
                right = LinearAttentionConfig(int(r["heads"]), int(r["dim"]), int(r["vdim"]), [float(x) for x in r["decay"]])
                if left.heads % left.kv_heads or left.rot_dims % 2 or left.rot_dims > left.dim:
                    raise ValueError("parallel: kv_heads must divide heads; rot.dims even and at most dim")
                if len(right.decay) != right.heads:
                    raise ValueError("parallel: the linear attention needs one decay per head")
                mc = ParallelConfig(left, right, float(m["left_scale"]), float(m["right_scale"]))
            else:
                raise ValueError(f"unknown layer type {kind!r}")
            mlp = L.get("mlp")
            if mlp is not None:
                if mlp.get("kind") != "dense":
                    raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
                mlp = FeedForwardConfig(int(mlp["ff"]), float(mlp["limit"]))
            layers.append(TiralixLayerConfig(kind, mc, mlp))
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   logit_scale=float(d.get("logit_scale", 1.0)), logit_softcap=float(d.get("logit_softcap") or 0.0),
                   layers=layers, eos_token_id=d.get("eos_token_id"))


def _default_layers():
    from ..layers import activation, gated_memory, linear_memory, row_norm_attention, stream

    class _L:
        stream_boundary = staticmethod(stream.stream_boundary)
        ScaledNorm = stream.ScaledNorm
        ConvBiasSilu = linear_memory.ConvBiasSilu
        SelectiveScan = linear_memory.SelectiveScan
        RowNormAttention = row_norm_attention.RowNormAttention
        JoinGated = row_norm_attention.JoinGated
        FixedDecayMemory = gated_memory.FixedDecayMemory
        ClampedGLU = activation.ClampedGLU
        ScaledSoftcap = activation.ScaledSoftcap
    return _L


# ------------------------------------------------------------------------------------------------ mixers
class TiralixSelectiveScan(nn.Module):
    def __init__(self, m: SelectiveScanConfig, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.m = m
        self.inp = _linear(width, 2 * m.inner, False, dtype, device)
        self.conv = L.ConvBiasSilu(m.inner, m.conv, device=device)
        self.x = _linear(m.inner, m.dt_rank + 2 * m.state, False, dtype, device)
        self.dt = _linear(m.dt_rank, m.inner, False, dtype, device)
        self.scan = L.SelectiveScan(m.inner, m.state, device=device)
        self.o = _linear(m.inner, width, False, dtype, device)

    def cache_specs(self):
        return [SlotStateSpec({"conv": ((self.m.conv - 1, self.m.inner), None), **self.scan.state_shapes()})]

    def names(self, p, t):
        return {p + "in": t + "inp.weight", p + "conv": t + "conv.weight", p + "conv.b": t + "conv.bias", p + "x": t + "x.weight",
                p + "dt": t + "dt.weight", p + "dt.b": t + "scan.dt_bias", p + "A_log": t + "scan.A_log", p + "D": t + "scan.D",
                p + "o": t + "o.weight"}

    def place(self, p, take):
        pass

    def finalize(self):
        self.scan.finalize()

    def forward(self, h, positions, caches):
        m, cache = self.m, caches[0]
        x, z = self.inp(h).split(m.inner, dim=1)
        x = self.conv(x, cache["conv"])
        dt, B, C = self.x(x).split((m.dt_rank, m.state, m.state), dim=1)
        return self.o(self.scan(x, self.dt(dt), z, B, C, cache["state"]))


class TiralixParallel(nn.Module, _FusedInputs):
    # the attention's and the memory's projections of the one input; the one-row-per-head gate comes last
    _inputs = ("lq", "lk", "lv", "rq", "rk", "rv", "rg", "lg")

    def __init__(self, m: ParallelConfig, width: int, eps: float, L, dtype, device):
        super().__init__()
        self.m = m
        a, r = m.left, m.right
        for name, rows in (("lq", a.heads * a.dim), ("lk", a.kv_heads * a.dim), ("lv", a.kv_heads * a.vdim), ("lg", a.heads),
                           ("rq", r.heads * r.dim), ("rk", r.heads * r.dim), ("rv", r.heads * r.vdim), ("rg", r.heads * r.vdim)):
            setattr(self, name, _linear(width, rows, False, dtype, device))
        self.left_cols, self.right_cols = a.heads * a.vdim, r.heads * r.vdim
        self.o = _linear(self.left_cols + self.right_cols, width, False, dtype, device)        # [left | right] columns
        self.attn = L.RowNormAttention(a.heads, a.kv_heads, a.dim, a.vdim, a.scale, eps, a.rot_dims, a.rot_base, a.rot_scaling,
                                       device=device)
        self.memory = L.FixedDecayMemory(r.heads, r.dim, r.vdim, r.decay, device=device)
        self.join = L.JoinGated(self.right_cols, eps, m.left_scale, m.right_scale, device=device)

    def cache_specs(self):
        a = self.m.left
        return [PagedKVSpec(a.kv_heads, a.dim, a.vdim), SlotStateSpec(self.memory.state_shapes())]

    def names(self, p, t):
        n = {p + "left." + x: t + f"l{x}.weight" for x in ("q", "k", "v", "g")}
        n.update({p + "right." + x: t + f"r{x}.weight" for x in ("q", "k", "v", "g")})
        n.update({p + "left.q.norm": t + "attn.q_norm", p + "left.k.norm": t + "attn.k_norm", p + "right.norm": t + "join.norm_weight"})
        return n

    def place(self, p, take):
        for name, cols in (("left.o", slice(0, self.left_cols)), ("right.o", slice(self.left_cols, None))):
            t = take(p + name)
            if t.shape != self.o.weight[:, cols].shape:
                raise ValueError(f"{p}{name}: shape {tuple(t.shape)} does not match the configuration")
            self.o.weight[:, cols].copy_(t)

    def finalize(self):
        self._fuse(self._inputs, multiple=8)

    def forward(self, h, positions, caches):
        a, r = self.m.left, self.m.right
        lq, lk, lv, rq, rk, rv, rg, lg = self._project(h, self._inputs)
        o = self.attn(lq.unflatten(1, (a.heads, a.dim)), lk.unflatten(1, (a.kv_heads, a.dim)), lv.unflatten(1, (a.kv_heads, a.vdim)),
                      positions, caches[0][0], caches[0][1])
        mem = self.memory(rq.unflatten(1, (r.heads, r.dim)), rk.unflatten(1, (r.heads, r.dim)), rv.unflatten(1, (r.heads, r.vdim)),
                          caches[1])
        return self.o(self.join(o, lg, mem, rg))


# ------------------------------------------------------------------------------------------------ layers
class TiralixFeedForward(nn.Module):
    def __init__(self, c: FeedForwardConfig, width: int, L, dtype, device):
        super().__init__()
        self.gate_up = _linear(width, 2 * c.ff, False, dtype, device)          # gate rows, then up rows
        self.down = _linear(c.ff, width, False, dtype, device)
        self.act = L.ClampedGLU(c.limit)

    def place(self, p, take):
        ff = self.down.weight.shape[1]
        for name, rows in (("gate", slice(0, ff)), ("up", slice(ff, None))):
            t = take(p + name)
            if t.shape != self.gate_up.weight[rows].shape:
                raise ValueError(f"{p}{name}: shape {tuple(t.shape)} does not match the configuration")
            self.gate_up.weight[rows].copy_(t)

    def forward(self, h):
        return self.down(self.act(self.gate_up(h)))


class TiralixLayer(nn.Module):
    def __init__(self, lc: TiralixLayerConfig, cfg: TiralixConfig, L, dtype, device):
        super().__init__()
        W = cfg.hidden_size
        kind = TiralixSelectiveScan if lc.kind == "mamba1" else TiralixParallel
        self.mix = kind(lc.mixer, W, cfg.norm_eps, L, dtype, device)
        self.norm1 = L.ScaledNorm(W, device=device)
        self.mlp = TiralixFeedForward(lc.mlp, W, L, dtype, device) if lc.mlp is not None else None
        self.norm2 = L.ScaledNorm(W, device=device) if lc.mlp is not None else None


class TiralixForCausalLM(nn.Module):
    #: the in-tree library this model's layers need (`nanovllm_amd._lib.build(target)`)
    kernel_library = "mixers"
    #: a cached prompt prefix cannot be taken over: the carried state at its end is not kept
    prefix_caching = False

    def __init__(self, cfg: TiralixConfig, layers=None, dtype: torch.dtype = torch.bfloat16, device=None):
        super().__init__()
        L = layers if layers is not None else _default_layers()
        self.config, self.dtype, self._L = cfg, dtype, L
        self.embed = nn.Embedding(cfg.vocab_size, cfg.hidden_size, dtype=dtype, device=device)
        self.layers = nn.ModuleList(TiralixLayer(lc, cfg, L, dtype, device) for lc in cfg.layers)
        self.final_norm = nn.Parameter(torch.ones(cfg.hidden_size, dtype=torch.float32, device=device))
        self.logits = L.ScaledSoftcap(cfg.logit_scale, cfg.logit_softcap)
        self._caches = None

    # ---- weights ----------------------------------------------------------------------------------------
    def checkpoint_names(self) -> dict[str, str]:
        """checkpoint tensor name -> parameter name of this module tree (the output projections of a parallel mixer and the two
        input projections of a feed-forward are placed separately)."""
        names = {"embed": "embed.weight", "final.norm": "final_norm"}
        for i, layer in enumerate(self.layers):
            p, t = f"l{i}.", f"layers.{i}."
            names.update({p + "norm1": t + "norm1.weight", p + "ls1": t + "norm1.scale"})
            names.update(layer.mix.names(p + "mix.", t + "mix."))
            if layer.mlp is not None:
                names.update({p + "norm2": t + "norm2.weight", p + "ls2": t + "norm2.scale", p + "mlp.down": t + "mlp.down.weight"})
        return names

    def load_tensors(self, tensors: dict[str, torch.Tensor]) -> None:
        """Copy checkpoint tensors (by checkpoint name) into the parameters.  The two output projections of a parallel mixer
        become the columns of one product, gate and up of a feed-forward the rows of one."""
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
                    layer.mlp.place(f"l{i}.mlp.", take)
            for ck, pn in names.items():
                t, prm = take(ck), params[pn]
                if t.shape != prm.shape:
                    raise ValueError(f"{ck}: checkpoint shape {tuple(t.shape)} != parameter {tuple(prm.shape)}")
                prm.copy_(t)
        extra = sorted(set(tensors) - seen)
        if extra:
            raise KeyError(f"checkpoint has tensors the model does not know, e.g. {extra[:3]}")
        self.finalize()

    def finalize(self) -> "TiralixForCausalLM":
        for layer in self.layers:
            layer.mix.finalize()
            layer.norm1.finalize()
            if layer.norm2 is not None:
                layer.norm2.finalize()
        return self

    # ---- caches -------------------------------------------------------------------------------------------
    def cache_specs(self) -> list:
        """Per layer the mixer's own: the convolution's carried inputs and the scan's state, or a paged KV cache and the
        linear attention's state."""
        return [spec for layer in self.layers for spec in layer.mix.cache_specs()]

    def bind_caches(self, caches: list) -> None:
        at, bound = 0, []
        for layer in self.layers:
            n = len(layer.mix.cache_specs())
            bound.append(caches[at:at + n])
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
        eps = cfg.norm_eps
        ctx = get_context()
        h = self.embed(input_ids)
        # the stream; what the sublayers read is the stream itself, in the matmul dtype (in a float32 model one tensor: a
        # sublayer has read it when the boundary behind it updates it)
        x = h.float() if dt != torch.float32 else h

        def add(y, norm, last):
            if last:
                return L.stream_boundary(x, normed=y, normed_weight=norm.applied, norm=self.final_norm, eps=eps, out_dtype=dt)[1]
            out = L.stream_boundary(x, normed=y, normed_weight=norm.applied, eps=eps, copy_dtype=dt if dt != torch.float32 else None)
            return x if out is None else out

        n = len(self.layers)
        for i, layer in enumerate(self.layers):
            ctx.layer_idx = i
            y = layer.mix(h, positions, self._caches[i])
            if i == n - 1 and logits_rows is not None and streams is None:
                # behind the last mixer only the asked rows go on: the caches and states of this step are complete
                x, y, logits_rows = x[logits_rows], y[logits_rows], None
            h = add(y, layer.norm1, i == n - 1 and layer.mlp is None)
            if layer.mlp is not None:
                h = add(layer.mlp(h), layer.norm2, i == n - 1)
            if streams is not None:
                streams.append(x.clone())
        if logits_rows is not None:
            h = h[logits_rows]
        return self.logits(F.linear(h, self.embed.weight))
