"""GPU parity of the HIP layers Nekodra is built from against their eager stand-ins (oracle/ref_nekodra_modules.py), layer by
layer, in float32 and bfloat16: widths on and off the vector path, one to sixteen column pieces per thread, odd strides,
identity experts whose rows nobody writes, per-head products with tails in every dimension, latent ranks on and off the
attention's tile sizes, pages that others left behind."""
import pytest
import torch

import nanovllm_amd as nv
from buvalix_util import paged_context
from oracle import ref_nekodra_modules as R

pytestmark = pytest.mark.gpu
DEV = "cuda"


def hip_layers():
    from nanovllm_amd.model.nekodra import _default_layers
    return _default_layers()


def rel(a, b):
    return ((a.float() - b.float()).norm() / b.float().norm().clamp_min(1e-30)).item()


def tol(dt):
    return 3e-6 if dt == torch.float32 else 1e-2


@pytest.fixture(params=[torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def dt(request):
    return request.param


def rn(g, *s, std=1.0, mean=0.0):
    return (torch.randn(*s, generator=g) * std + mean).to(DEV)


def pair(cls_name, *args, **kw):
    a, b = getattr(hip_layers(), cls_name)(*args, device=DEV, **kw), getattr(R, cls_name)(*args, device=DEV, **kw)
    g = torch.Generator().manual_seed(len(cls_name))
    with torch.no_grad():
        for (_, pa), (_, pb) in zip(a.named_parameters(), b.named_parameters()):
            v = rn(g, *pa.shape, std=0.3, mean=0.2).to(pa.dtype)
            pa.copy_(v), pb.copy_(v)
    return a, b


@pytest.mark.parametrize("W", [7, 96, 100, 521, 1500, 2048, 5000, 9001, 16384])
def test_two_layer_norms_behind_routed_and_added_parts(dt, W):
    L, g, T, n, E = hip_layers(), torch.Generator().manual_seed(W), 9, 3, 5
    x, a1, a2 = rn(g, T, W, mean=2.0), rn(g, T, W).to(dt), rn(g, T, W + 3).to(dt)[:, :W]
    through, parts = rn(g, T, W).to(dt), rn(g, T, n, W)
    ids = torch.stack([torch.randperm(E + 2, generator=g)[:n] for _ in range(T)]).to(torch.int32)
    ids[0], ids[1] = torch.tensor([5, 6, 0]), torch.tensor([0, 1, 2])
    ids, wts = ids.to(DEV), torch.rand(T, n, generator=g).to(DEV)
    parts[ids >= E] = float("nan")                       # what nobody wrote must not be read
    na, nb = (rn(g, W, std=0.3, mean=1.0), rn(g, W)), (rn(g, W, std=0.3, mean=1.0), rn(g, W))
    xa, xb = x.clone(), x.clone()
    kw = dict(adds=[a1, a2], routed=(parts, ids, wts, E, through), norm_a=na, norm_b=nb, eps=1e-6, out_dtype=dt, want_f32_b=True)
    A, B = L.layernorm_pair_boundary(xa, **kw), R.layernorm_pair_boundary(xb, **kw)
    assert torch.isfinite(xa).all() and rel(xa, xb) < 3e-6 and rel(A[2], B[2]) < 3e-6
    assert rel(A[0], B[0]) < tol(dt) and rel(A[1], B[1]) < tol(dt)
    kw = dict(adds=[a1], norm_a=na, eps=1e-6, out_dtype=dt)
    A, B = L.layernorm_pair_boundary(xa, **kw), R.layernorm_pair_boundary(xb, **kw)
    assert A[1] is None and A[2] is None and rel(xa, xb) < 3e-6 and rel(A[0], B[0]) < tol(dt)
    before = xa.clone()
    A, B = (M.layernorm_pair_boundary(xx, norm_a=na, norm_b=nb, eps=1e-6, out_dtype=dt) for M, xx in ((L, xa), (R, xb)))
    assert torch.equal(before, xa) and A[2] is None and rel(A[0], B[0]) < tol(dt) and rel(A[1], B[1]) < tol(dt)


def test_variance_of_a_row_far_from_zero(dt):
    """A mean a thousand times the spread: deviations are squared, not the raw values."""
    L, g, W = hip_layers(), torch.Generator().manual_seed(1), 640
    x = rn(g, 4, W, mean=1000.0)
    one, zero = torch.ones(W, device=DEV), torch.zeros(W, device=DEV)
    a, _, _ = L.layernorm_pair_boundary(x, norm_a=(one, zero), eps=1e-6, out_dtype=torch.float32)
    d = x.double() - x.double().mean(-1, keepdim=True)
    assert rel(a, d / (d.pow(2).mean(-1, keepdim=True) + 1e-6).sqrt()) < 1e-4


def test_position_embedding(dt):
    a, b = pair("PositionEmbedding", 31, 17, 50, dtype=dt)
    ids, pos = torch.tensor([0, 30, 5, 5], device=DEV), torch.tensor([0, 16, 3, 4], device=DEV)
    assert torch.equal(a(ids, pos), b(ids, pos))


@pytest.mark.parametrize("cols,stride", [(64, 128), (100, 200), (33, 66), (8, 19), (2048, 4096)])
def test_silu_and_mul(dt, cols, stride):
    L, g = hip_layers(), torch.Generator().manual_seed(cols)
    x = rn(g, 7, stride, std=3.0).to(dt)[:, :2 * cols]
    assert rel(L.SiluAndMulRows()(x), R.SiluAndMulRows()(x)) < tol(dt)


@pytest.mark.parametrize("T,H,K,N", [(1, 3, 10, 18), (5, 2, 64, 128), (70, 4, 33, 65), (300, 1, 128, 256), (17, 5, 48, 20),
                                     (2100, 8, 96, 40), (4000, 16, 128, 128)])
@pytest.mark.parametrize("gated", [False, True], ids=["plain", "gated"])
def test_per_head_products(dt, T, H, K, N, gated):
    a, b = pair("HeadLinear", H, K, N, dtype=dt)
    g = torch.Generator().manual_seed(T + K)
    x = rn(g, T, H * K + 8).to(dt)[:, :H * K]
    z = rn(g, T, H * N + 5, std=3.0).to(dt)[:, 5:] if gated else None
    assert rel(a(x, z), b(x, z)) < tol(dt)


N_Q, N_K = [5, 1, 70, 2, 1], [5, 140, 90, 2, 9]


@pytest.mark.parametrize("H,rank,own", [(3, 18, True), (5, 64, True), (16, 128, True), (2, 256, True), (1, 512, True), (9, 40, True),
                                        (20, 96, False), (4, 7, True), (33, 32, False)])
def test_latent_attention_with_a_sink(dt, H, rank, own):
    ctx, _ = paged_context(N_Q, N_K, 8, 60, 1, DEV)
    nv.set_context(ctx)
    T = sum(N_Q)
    a, b = pair("UnrotatedLatentAttention", H, rank, 2.0 / rank ** 0.5, 1e-6, own_latent=own, use_sink=True)
    with torch.no_grad():
        for m in (a, b):
            m.sink.copy_(torch.linspace(-3.0, 5.0, H))
    g = torch.Generator().manual_seed(H * rank)
    q, raw = rn(g, T, H * rank).to(dt), rn(g, T, rank + 4).to(dt)[:, :rank]
    ka = rn(g, 60, 8, 1, rank).to(dt)                     # stale pages
    kb = ka.clone()
    ya, yb = a(q, raw if own else None, ka, ka[..., :rank]), b(q, raw if own else None, kb, kb[..., :rank])
    nv.set_context(None)
    assert rel(ya, yb) < tol(dt) and rel(ka, kb) < tol(dt)
    if not own:
        assert torch.equal(ka, kb)


@pytest.mark.parametrize("E,top", [(8, 2), (6, 6), (1, 1), (20, 3), (70, 20), (130, 8), (1024, 40)])
def test_softmax_routing_with_a_correction(E, top):
    a, b = pair("SoftmaxRouter", E, top, 2.25)
    g = torch.Generator().manual_seed(E)
    with torch.no_grad():
        c = rn(g, E, std=0.05, mean=-0.5)                 # choice values below zero
        a.correction.copy_(c), b.correction.copy_(c)
    logits = rn(g, 77, E, std=2.0)
    (ia, wa), (ib, wb) = a(logits), b(logits)
    assert ia.sort(1).values.tolist() == ib.sort(1).values.tolist()
    assert rel(wa.gather(1, ia.long().argsort(1)), wb.gather(1, ib.long().argsort(1))) < 1e-6
    a.correction = b.correction = None
    (ia, wa), (ib, wb) = a(logits), b(logits)
    assert torch.equal(ia, ib) and rel(wa, wb) < 1e-6


@pytest.mark.parametrize("T,W,E,extra,top,ff", [(26, 40, 5, 2, 3, 12), (300, 64, 4, 1, 3, 32), (9, 100, 40, 9, 4, 20), (1, 24, 3, 2, 1, 7),
                                                (700, 96, 6, 3, 4, 64)])
def test_silu_experts_leave_identity_choices_alone(dt, T, W, E, extra, top, ff):
    a, b = hip_layers().SiluExperts(), R.SiluExperts()
    g = torch.Generator().manual_seed(T)
    h, gu, down = rn(g, T, W).to(dt), rn(g, E, 2 * ff, W, std=0.3).to(dt), rn(g, E, W, ff, std=0.3).to(dt)
    ids = torch.stack([torch.randperm(E + extra, generator=g)[:top] for _ in range(T)]).to(torch.int32).to(DEV)
    if T == 1:
        ids.fill_(E)                                      # no product at all in the step
    w = torch.rand(T, top, generator=g).to(DEV)
    ya, yb = a(h, ids, w, gu, down), b(h, ids, w, gu, down)
    use = ids < E
    assert not use.any() or rel(ya[use], yb[use]) < tol(dt)
