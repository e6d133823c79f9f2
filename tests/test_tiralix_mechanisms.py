"""Each Tiralix mechanism alone, against the plain functions of oracle/ref_tiralix.py, on inputs made so that a fault
shows: the model's own modules (built on the eager stand-in layers on the CPU and, marked gpu, on the HIP kernels in
float32, where noted also in bfloat16) are driven step by step through a paged cache with stale pages and state slots that
others used before, and compared with the oracle's whole-sequence result.

  * attention: a peaked softmax (large score scale) so that one missing or misplaced key moves the output; one far key, the
    first key, keys on page borders that a query is aimed at; norms over the whole row (heads of very different size); rotary
    frequencies kept, blended and stretched, with their magnitude; gates that differ from head to head;
  * linear attention: a first token read hundreds of tokens later through a decay close to one, a decay of zero (only the
    token itself), portions on both sides of every launch's limits; the norm over all heads together;
  * selective scan: a first token written with a large step and kept by tiny ones, read hundreds of tokens later; steps beyond
    the softplus' linear range; convolution taps that reach across portions and in front of the sequence's start;
  * the clamps of the feed-forward (the gate's has no lower side), the boundary, the logits' cap."""
import math

import pytest
import torch

from nanovllm_amd.model import tiralix as M
from oracle import ref_tiralix as O
from test_divadra_mechanisms import close, rn, run_in_steps
from tiralix_util import layer_namespace, mamba_tensors, parallel_tensors

BACKENDS = [pytest.param("cpu", id="cpu"), pytest.param("cuda", id="gpu", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16


@pytest.fixture(params=BACKENDS)
def dev(request):
    return request.param


def lin(g, o, i, gain=1.0):
    return rn(g, o, i, std=gain / math.sqrt(i))


def mixer(kind, m, w, W, dev, dtype=F32, eps=1e-5):
    """The model's mixer module with checkpoint-named tensors `w` (no prefix)."""
    cfg = M.TiralixConfig.from_dict({"vocab": 4, "width": W, "norm": {"eps": eps}, "layers": [{"type": kind, "mixer": m, "mlp": None}]})
    cls = M.TiralixSelectiveScan if kind == "mamba1" else M.TiralixParallel
    mod = cls(cfg.layers[0].mixer, W, eps, layer_namespace(dev), dtype, dev)
    params, seen = dict(mod.named_parameters()), set()

    def take(name):
        seen.add(name)
        return w[name]
    with torch.no_grad():
        mod.place("", take)
        for ck, pn in mod.names("", "").items():
            params[pn].copy_(take(ck))
    assert seen == set(w), set(w) ^ seen
    mod.finalize()
    return mod


def caches_of(mod, dev, dtype=F32, nb=80, bs=4):
    """Cache pages and slots as other owners left them."""
    out = []
    for spec in mod.cache_specs():
        if hasattr(spec, "kv_heads"):
            out.append((torch.randn(nb, bs, spec.kv_heads, spec.key_dim, device=dev).to(dtype),
                        torch.randn(nb, bs, spec.kv_heads, spec.value_dim, device=dev).to(dtype)))
        else:
            out.append({n: torch.randn(4, *shape, device=dev).to(dt or dtype) for n, (shape, dt) in spec.tensors.items()})
    return out


def drive(mod, h, portions, dev, other=None, dtype=F32, nb=80):
    caches = caches_of(mod, dev, dtype, nb)
    return run_in_steps(lambda x, pos: mod(x.to(dtype), pos, caches), h, portions, dev, num_blocks=nb, other=other)


def parallel(g, W, left, right, left_scale=1.0, right_scale=1.0):
    m = {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}
    w = parallel_tensors(g, m, W, lambda *s, **k: rn(g, *s, **k), lambda *a: lin(g, *a))
    return m, w


RIGHT = {"heads": 2, "dim": 5, "vdim": 4, "decay": [0.5, 0.95]}
LEFT = {"heads": 2, "kv_heads": 1, "dim": 6, "vdim": 5, "scale": 0.4}


# ------------------------------------------------------------------------------------------------ attention
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot", [
    (4, 2, 16, 8, {"dims": 16, "base": 40.0, "scaling": {"factor": 5.0, "original": 400, "fast": 32.0, "slow": 8.0}}),
    (3, 1, 10, 13, {"dims": 10, "base": 500.0}), (2, 2, 6, 6, None),
    (9, 1, 12, 4, {"dims": 4, "base": 9.0, "scaling": {"factor": 3.0, "original": 2, "fast": 0.5, "slow": 0.4}}),
    (2, 1, 16, 32, {"dims": 8, "base": 1e4, "scaling": {"factor": 16.0, "original": 64, "fast": 32.0, "slow": 1.0}})])
def test_attention_peaked_softmax_every_key_counts(dev, heads, kv_heads, dim, vdim, rot):
    """Score scale 5 / sqrt(dim): a few keys carry each row, so a key that is lost, shifted by one or rotated by a wrong
    frequency moves the output far beyond the bound.  Pages of 4, portions that cut pages.  The right side is switched off."""
    g = torch.Generator().manual_seed(3 + heads)
    W, T = 24, 150
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 5.0 / math.sqrt(dim)}
    if rot:
        left["rot"] = rot
    m, w = parallel(g, W, left, RIGHT, left_scale=1.4, right_scale=0.0)
    if rot and rot["dims"] == 16:
        f0, one = O.rotary_frequencies({"dims": 16, "base": 40.0})
        f1, mag = O.rotary_frequencies(rot)
        assert one == 1.0 and abs(mag - (0.1 * math.log(5.0) + 1.0)) < 1e-12
        kept, stretched = f1 == f0, (f1 - f0 / 5.0).abs() < 1e-8
        assert kept.any() and stretched.any() and (~kept & ~stretched).any()
    h, other = rn(g, T, W), rn(g, 12, W)
    want = O.parallel_mixer(m, w, "", h, 1e-5)
    assert (want - 1.4 * O.gated_attention(left, w, "left.", h, 1e-5)).abs().max() < 1e-5
    if rot and rot.get("scaling"):
        plain = O.gated_attention({**left, "rot": {"dims": rot["dims"], "base": rot["base"]}}, w, "left.", h, 1e-5) * 1.4
        assert (want - plain).norm() > 0.05 * want.norm()
    mod = mixer("parallel", m, w, W, dev)
    for portions in ([T], [1], [2, 3, 1, 1, 64, 2, 70], [5, 3]):
        close(drive(mod, h, portions, dev, other), want)


@pytest.mark.parametrize("target,query,portions", [(0, 299, [1]), (3, 299, [296, 1]), (4, 298, [300]), (131, 260, [128, 4, 1]),
                                                    (299, 299, [7, 1]), (63, 64, [64, 1])])
@pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
def test_attention_a_far_key(dev, target, query, portions, dtype):
    """Identity-like projections (the input row IS [q | k | v]); query and target key are aligned, every other score is small:
    the first head's output is the target's value.  The key and value size (64, 32) take the tile and decode kernels."""
    if dtype == BF16 and dev == "cpu":
        pytest.skip("the kernels' own precision")
    g = torch.Generator().manual_seed(5)
    H, G, D, Dv, T = 2, 1, 64, 32, 300
    W = (H + G) * D + Dv
    left = {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "scale": 12.0 / D}
    m, w = parallel(g, W, left, RIGHT, right_scale=0.0)
    eye = torch.eye(W)
    w["left.q"], w["left.k"], w["left.v"] = eye[:H * D], eye[H * D:(H + G) * D], eye[(H + G) * D:]
    w["left.q.norm"], w["left.k.norm"] = torch.ones(H * D), torch.full((D,), 2.0)
    w["left.g"] = torch.zeros(H, W)                                       # every gate one half
    w["left.o"][:, Dv:] = 0.0                                             # only head 0 is looked at
    aim = torch.where(torch.rand(D, generator=g) < 0.5, -1.0, 1.0)
    away = aim * torch.where(torch.arange(D) % 2 == 0, -1.0, 1.0)          # orthogonal to aim
    h = rn(g, T, W, std=0.2)
    h[:, H * D:(H + G) * D] += 3.0 * away
    h[target, H * D:(H + G) * D] = 3.0 * aim
    h[query, :D] = 3.0 * aim
    h[:, (H + G) * D:] = rn(g, T, Dv)
    h = h.to(dtype).float()
    w = {k: v.to(dtype).float() for k, v in w.items()}
    want = O.parallel_mixer(m, w, "", h, 1e-5)
    only = O.linear(torch.cat([0.5 * h[target, (H + G) * D:], torch.zeros(Dv)]), w["left.o"])
    assert (want[query] - only).norm() < 0.02 * only.norm()                # head 0 reads the target
    mod = mixer("parallel", m, w, W, dev, dtype)
    got = drive(mod, h, portions, dev, rn(g, 5, W), dtype, nb=160)
    close(got, want, 2e-5 if dtype == F32 else 2e-2)
    close(got[query], want[query], 2e-5 if dtype == F32 else 2e-2)


def test_attention_norm_spans_all_heads_and_gates_are_per_head(dev):
    """Head 0 projects to values a hundred times those of head 1: a norm per head would lift head 1 to the same size.  Gates
    of one head far open, the others shut to different degrees."""
    g = torch.Generator().manual_seed(6)
    W, T = 20, 40
    left = {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 6, "scale": 2.0, "rot": {"dims": 4, "base": 30.0}}
    m, w = parallel(g, W, left, RIGHT, right_scale=0.0)
    for n, hd in (("left.q", 4), ("left.k", 2)):
        w[n].view(hd, 8, W)[0] *= 100.0
    w["left.g"] *= torch.tensor([8.0, 1.0, 0.1, 4.0])[:, None]
    h = rn(g, T, W)
    want = O.parallel_mixer(m, w, "", h, 1e-5)
    swapped = O.parallel_mixer(m, {**w, "left.g": w["left.g"].flip(0)}, "", h, 1e-5)
    assert (want - swapped).norm() > 0.2 * want.norm()
    mod = mixer("parallel", m, w, W, dev)
    for portions in ([T], [1], [9, 2]):
        close(drive(mod, h, portions, dev, rn(g, 4, W)), want)


# ------------------------------------------------------------------------------------------------ linear attention
@pytest.mark.parametrize("heads,dim,vdim", [(3, 10, 6), (1, 64, 64), (2, 33, 70)])
@pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
def test_linear_attention_reads_a_first_token_hundreds_of_tokens_later(dev, heads, dim, vdim, dtype):
    """A large first token; the decay of head 0 is 0.9995, so it is still there 260 tokens on, in portions on both sides of 16
    (token by token / chunks), 64 (one chunk) and 256 tokens.  The left side is switched off."""
    if dtype == BF16 and dev == "cpu":
        pytest.skip("the kernels' own precision")
    g = torch.Generator().manual_seed(7)
    W, T = 20, 330
    right = {"heads": heads, "dim": dim, "vdim": vdim, "decay": [0.9995, 0.9, 0.0][:heads]}
    m, w = parallel(g, W, LEFT, right, left_scale=0.0, right_scale=0.7)
    h = rn(g, T, W, std=0.5)
    h[0] *= 8.0
    h, w = h.to(dtype).float(), {k: v.to(dtype).float() for k, v in w.items()}
    want = O.parallel_mixer(m, w, "", h, 1e-5)
    lost = O.parallel_mixer(m, w, "", torch.cat([torch.zeros(1, W), h[1:]]), 1e-5)
    assert (want[-1] - lost[-1]).norm() > 0.05 * want[-1].norm()           # the last row does depend on the first token
    mod = mixer("parallel", m, w, W, dev, dtype)
    for portions in ([T], [1], [2, 327, 1], [15, 16, 17, 2, 63, 64, 65], [257, 1, 72], [17]):
        got = drive(mod, h, portions, dev, rn(g, 9, W), dtype, nb=170)
        close(got, want, 2e-5 if dtype == F32 else 1.5e-2)
        close(got[-1], want[-1], 5e-5 if dtype == F32 else 3e-2)


def test_linear_attention_decay_of_zero_and_norm_over_all_heads(dev):
    """decay 0: o_t = (k_t . q_t) v_t, whatever came before; decay 1: a plain sum.  The heads differ by orders of magnitude, so
    a norm per head would be another function."""
    g = torch.Generator().manual_seed(8)
    W, T = 16, 90
    right = {"heads": 2, "dim": 6, "vdim": 8, "decay": [0.0, 1.0]}
    m, w = parallel(g, W, LEFT, right, left_scale=0.0)
    h = rn(g, T, W)
    silu = lambda n, d: O.silu(O.linear(h, w["right." + n])).view(T, 2, d)
    q, k, v = silu("q", 6), silu("k", 6), silu("v", 8)
    o = O.decayed_memory(q, k, v, torch.tensor([0.0, 1.0]))
    close(o[:, 0], (q[:, 0] * k[:, 0]).sum(-1, keepdim=True) * v[:, 0], 1e-6)
    close(o[40, 1], (k[:41, 1].t() @ v[:41, 1]).t() @ q[40, 1], 1e-5)
    want = O.parallel_mixer(m, w, "", h, 1e-5)
    mod = mixer("parallel", m, w, W, dev)
    for portions in ([T], [1], [20, 1, 40]):
        close(drive(mod, h, portions, dev, rn(g, 6, W)), want)


@pytest.mark.parametrize("left_scale,right_scale", [(1.0, 1.0), (0.3, 1.9), (-0.5, 0.2)])
def test_parallel_sides_are_added_with_their_factors(dev, left_scale, right_scale):
    g = torch.Generator().manual_seed(9)
    W, T = 24, 30
    m, w = parallel(g, W, LEFT, RIGHT, left_scale, right_scale)
    h = rn(g, T, W)
    want = left_scale * O.gated_attention(LEFT, w, "left.", h, 1e-5) + right_scale * O.lightning_attention(RIGHT, w, "right.", h, 1e-5)
    mod = mixer("parallel", m, w, W, dev)
    close(drive(mod, h, [4, 18, 1], dev, rn(g, 6, W)), want)


# ------------------------------------------------------------------------------------------------ selective scan
@pytest.mark.parametrize("inner,state,dt_rank,conv", [(12, 5, 3, 4), (40, 16, 1, 1), (9, 33, 7, 6), (64, 4, 8, 2)])
def test_selective_scan_keeps_a_first_token(dev, inner, state, dt_rank, conv):
    """Tiny step sizes and slow rates keep what a first token with large steps has written for 260 tokens."""
    g = torch.Generator().manual_seed(10 + inner)
    W, T = 20, 260
    m = {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}
    w = mamba_tensors(g, m, W, lambda *s, **k: rn(g, *s, **k), lambda *a: lin(g, *a))
    w["dt.b"], w["A_log"] = rn(g, inner, std=0.5, mean=-5.0), rn(g, inner, state, std=0.5, mean=-0.7)
    h = rn(g, T, W, std=0.5)
    h[0] *= 10.0
    want = O.mamba_mixer(m, w, "", h)
    lost = O.mamba_mixer(m, w, "", torch.cat([torch.zeros(1, W), h[1:]]))
    assert (want[-1] - lost[-1]).norm() > 0.02 * want[-1].norm()
    mod = mixer("mamba1", m, w, W, dev)
    for portions in ([T], [1], [2, 255, 1], [129, 2, 64], [3, 16, 17, 15]):
        got = drive(mod, h, portions, dev, rn(g, 9, W), nb=140)
        close(got, want)
        close(got[-1], want[-1], 5e-5)


def test_selective_scan_in_segments_keeps_a_first_token(dev):
    """The same over prompts long enough to be cut along time (at least 256 tokens of one sequence)."""
    g = torch.Generator().manual_seed(12)
    W, T = 12, 700
    m = {"inner": 24, "state": 6, "dt_rank": 2, "conv": 3}
    w = mamba_tensors(g, m, W, lambda *s, **k: rn(g, *s, **k), lambda *a: lin(g, *a))
    w["dt.b"], w["A_log"] = rn(g, 24, std=0.5, mean=-6.0), rn(g, 24, 6, std=0.5, mean=-0.7)
    h = rn(g, T, W, std=0.5)
    h[0] *= 10.0
    want = O.mamba_mixer(m, w, "", h)
    lost = O.mamba_mixer(m, w, "", torch.cat([torch.zeros(1, W), h[1:]]))
    assert (want[-1] - lost[-1]).norm() > 0.02 * want[-1].norm()
    mod = mixer("mamba1", m, w, W, dev)
    for portions in ([T], [1, 698, 1], [290, 410]):
        close(drive(mod, h, portions, dev, rn(g, 9, W), nb=360), want)


def test_selective_scan_steps_beyond_the_linear_range(dev):
    """dt_raw far above 20 (softplus is the identity) and far below (softplus is the exponential); rates that make the decay
    vanish and ones that leave it at one."""
    g = torch.Generator().manual_seed(13)
    W, T = 16, 50
    m = {"inner": 10, "state": 4, "dt_rank": 2, "conv": 2}
    w = mamba_tensors(g, m, W, lambda *s, **k: rn(g, *s, **k), lambda *a: lin(g, *a))
    w["dt.b"] = torch.linspace(-40.0, 40.0, 10)
    w["A_log"] = torch.linspace(-9.0, 4.0, 40).view(10, 4)
    h = rn(g, T, W)
    want = O.mamba_mixer(m, w, "", h)
    assert torch.isfinite(want).all()
    mod = mixer("mamba1", m, w, W, dev)
    for portions in ([T], [1], [7, 2]):
        close(drive(mod, h, portions, dev, rn(g, 4, W)), want)


# ------------------------------------------------------------------------------------------------ feed-forward, boundary, logits
def test_feed_forward_clamps(dev):
    """The gate is clamped from above only, the up branch on both sides; inputs far beyond the limit on every side."""
    L, g = layer_namespace(dev), torch.Generator().manual_seed(15)
    W, ff, T = 28, 50, 11
    w = {"gate": rn(g, ff, W, std=0.8), "up": rn(g, ff, W, std=0.8), "down": rn(g, W, ff, std=0.3)}
    mod = M.TiralixFeedForward(M.FeedForwardConfig(ff, 1.2), W, L, F32, dev)
    with torch.no_grad():
        mod.place("", lambda n: w[n])
        mod.down.weight.copy_(w["down"])
    h = rn(g, T, W, std=1.5)
    z = h @ w["gate"].t()
    assert (z > 1.2).any() and (z < -1.2).any()
    close(mod(h.to(dev)).cpu(), O.feed_forward({"kind": "dense", "ff": ff, "limit": 1.2}, w, "", h))
    both = O.linear(O.clamped_glu(z.clamp(min=-1.2), h @ w["up"].t(), 1.2), w["down"])
    assert (mod(h.to(dev)).cpu() - both).norm() > 1e-2 * both.norm()


def test_boundary_norms_the_output_not_the_stream_and_logits_are_capped(dev):
    L, g = layer_namespace(dev), torch.Generator().manual_seed(16)
    T, W = 9, 30
    norm = L.ScaledNorm(W, device=dev)
    nw, ls = rn(g, W, std=0.3, mean=1.0), rn(g, W, std=0.5)
    with torch.no_grad():
        norm.weight.copy_(nw), norm.scale.copy_(ls)
    norm.finalize()
    x, y, fw = rn(g, T, W, std=5.0), rn(g, T, W, std=1e-3), rn(g, W)
    xd = x.clone().to(dev)
    h = L.stream_boundary(xd, normed=y.to(dev), normed_weight=norm.applied, eps=1e-5, copy_dtype=F32)
    want = x + ls * O.rms_norm(y, nw, 1e-5)                                # eps counts: the output is small
    close(xd.cpu(), want, 1e-6)
    close(h.cpu(), want, 1e-6)
    _, h = L.stream_boundary(xd, normed=y.to(dev), normed_weight=norm.applied, norm=fw.to(dev), eps=1e-5, out_dtype=F32)
    want = want + ls * O.rms_norm(y, nw, 1e-5)
    close(h.cpu(), O.rms_norm(want, fw, 1e-5), 1e-6)
    z = rn(g, T, 50, std=40.0)
    got = L.ScaledSoftcap(0.5, 7.0)(z.to(dev)).cpu()
    close(got, 7.0 * torch.tanh(0.5 * z / 7.0), 1e-6)
    assert got.abs().max() <= 7.0
    close(L.ScaledSoftcap(0.5, 0.0)(z.to(dev)).cpu(), 0.5 * z, 1e-6)
