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
                                        (20, 96, False), (4, 7, True), (33, 32, False), (2, 640, True)])
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


def reference_rows(q, cache, ctx, scale, sink, Dv):
    """fp32 attention of q [T, H, D] over the cached rows, sequence by sequence, heads together."""
    cu_q, cu_k, bs = ctx.cu_seqlens_q.tolist(), ctx.cu_seqlens_k.tolist(), cache.shape[1]
    out = torch.zeros(q.shape[0], q.shape[1], Dv, device=q.device)
    for b in range(len(cu_q) - 1):
        nq, nk = cu_q[b + 1] - cu_q[b], cu_k[b + 1] - cu_k[b]
        pos = torch.arange(nk, device=q.device)
        rows = cache.view(-1, q.shape[2])[ctx.block_tables[b].long()[pos // bs] * bs + pos % bs].float()
        s = torch.matmul(q[cu_q[b]:cu_q[b + 1]].float(), rows.t()) * scale                      # [nq, H, nk]
        s = s.masked_fill((pos[None, :] > (nk - nq + torch.arange(nq, device=q.device))[:, None])[:, None], float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink.view(1, -1, 1).expand(nq, -1, 1)], dim=-1)
        out[cu_q[b]:cu_q[b + 1]] = torch.matmul(torch.softmax(s, dim=-1)[..., :nk], rows[:, :Dv])
    return out.reshape(q.shape[0], -1)


BUILT = [(32, 32), (64, 64), (96, 96), (128, 128), (160, 160), (192, 192), (224, 224), (256, 256), (320, 320), (384, 384), (512, 512), (160, 128),
         (192, 128), (256, 192), (320, 256), (576, 512)]
STEPS = {"mixed": ([5, 1, 200, 2, 1, 77], [5, 140, 333, 66, 1, 640]), "decode": ([1] * 5, [1, 32, 33, 700, 64]), "long_decode": ([1, 1], [5000, 2049]),
         "long_chunk": ([40], [3000]), "prompts": ([64, 63, 129], [64, 63, 129])}


@pytest.mark.parametrize("D,Dv", BUILT, ids=lambda n: str(n))
@pytest.mark.parametrize("step", sorted(STEPS))
def test_matrix_core_latent_attention(D, Dv, step):
    from nanovllm_amd import _lib, ops
    assert _lib.mixers().nv_attn_latent_ok(D, Dv, 64) == 1
    n_q, n_k = STEPS[step]
    for H, bs, sinks in ((16, 64, True), (3, 128, False)) if step != "mixed" else ((33, 64, True), (1, 192, True)):
        ctx, _ = paged_context(n_q, n_k, bs, sum(-(-n // bs) for n in n_k) + 3, D, DEV)
        g = torch.Generator().manual_seed(D + H)
        q = rn(g, sum(n_q), H, D, std=3.0 / D ** 0.5).to(torch.bfloat16)
        cache = rn(g, sum(-(-n // bs) for n in n_k) + 3, bs, 1, D).to(torch.bfloat16)
        sink = torch.linspace(-3.0, 6.0, H, device=DEV) if sinks else None
        got = ops.attn_latent_paged(q, cache, cache[..., :Dv], ctx.cu_seqlens_q, ctx.cu_seqlens_k, ctx.block_tables, 0.9, sink,
                                    max(n_q), max(n_k), -1)
        want = reference_rows(q, cache, ctx, 0.9, sink, Dv)
        assert torch.isfinite(got).all()
        err = (got.float() - want).view(sum(n_q), -1).norm(dim=-1) / want.norm(dim=-1)
        assert err.max().item() < 1.2e-2, (H, bs, int(err.argmax()), err.max().item())


@pytest.mark.parametrize("D", [64, 160, 512])
def test_matrix_core_latent_attention_finds_each_key(D):
    """Every query row is aimed at one key (the score stands 20 above the others): the key at the row's own position, ahead of
    it (which must weigh nothing), at tile and page edges, and where the launch cuts the keys into ranges."""
    from nanovllm_amd import ops
    n_q, n_k, H, bs = [200, 1, 1, 1], [1500, 1500, 4097, 65], 4, 64
    ctx, _ = paged_context(n_q, n_k, bs, 130, D, DEV)
    g = torch.Generator().manual_seed(D)
    T = sum(n_q)
    unit = torch.nn.functional.normalize(torch.randn(130 * bs, D, generator=g), dim=-1)
    cache = (unit * D ** 0.5).to(torch.bfloat16).view(130, bs, 1, D).to(DEV)
    targets, q = [], torch.zeros(T, H, D)
    cu_q = [0] + torch.tensor(n_q).cumsum(0).tolist()
    tables = ctx.block_tables.cpu()
    flat = cache.view(-1, D).float().cpu()
    for b in range(4):
        for i in range(n_q[b]):
            pos = n_k[b] - n_q[b] + i
            for h in range(H):
                edges = [pos, 0, 31, 32, 63, 64, 255, 256, 511, 512, 1023, 1024, pos - 1, pos + 1]
                t = edges[(i * H + h) % len(edges)]
                t = t if 0 <= t < n_k[b] else pos
                targets.append((b, t, pos))
                q[cu_q[b] + i, h] = flat[int(tables[b][t // bs]) * bs + t % bs] * (20.0 / D)
    got = ops.attn_latent_paged(q.to(torch.bfloat16).to(DEV), cache, cache[..., :D], ctx.cu_seqlens_q, ctx.cu_seqlens_k, ctx.block_tables, 1.0,
                                None, max(n_q), max(n_k), -1)
    want = reference_rows(q.to(torch.bfloat16).to(DEV), cache, ctx, 1.0, None, D)
    rows_got, rows_want = got.float().view(T * H, D), want.view(T * H, D)
    err = (rows_got - rows_want).norm(dim=-1) / rows_want.norm(dim=-1)
    seen = torch.tensor([t <= pos for _, t, pos in targets])
    assert err[seen.to(DEV)].max().item() < 1.2e-2, err.max().item()
    assert (rows_got - rows_want)[~seen.to(DEV)].abs().max().item() < 0.1
    for k, (b, t, pos) in enumerate(targets):
        own = flat[int(tables[b][t // bs]) * bs + t % bs]
        if t <= pos:
            assert torch.nn.functional.cosine_similarity(rows_got[k].cpu(), own, dim=0).item() > 0.9, (b, t, pos)
        else:
            assert (rows_got[k].cpu() - own).norm() > 0.3 * own.norm(), (b, t, pos)
