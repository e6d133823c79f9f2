"""GPU parity of the HIP layers Tiralix is built from against their eager stand-ins (oracle/ref_tiralix_modules.py), layer by
layer, in float32 and bfloat16, on a mixed step (prompt portions on both sides of every launch's limits beside single rows,
shuffled pages, state slots in any order, states and pages that others left behind) with sizes that exercise the kernels'
tails and their vector paths: widths that are and are not a multiple of a piece, odd strides, rotated parts of 2 to 128
dimensions, every number of lanes a channel of the scan may have, chunks with every padded key size."""
import pytest
import torch

import nanovllm_amd as nv
from buvalix_util import paged_context
from oracle import ref_tiralix_modules as R

pytestmark = pytest.mark.gpu
DEV = "cuda"


def hip_layers():
    from nanovllm_amd.model.tiralix import _default_layers
    return _default_layers()


def rel(a, b):
    assert torch.isfinite(a.float()).all()
    return ((a.float() - b.float()).norm() / b.float().norm().clamp_min(1e-30)).item()


def tol(dt):
    return 3e-6 if dt == torch.float32 else 1e-2


@pytest.fixture(params=[torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def dt(request):
    return request.param


N_Q, N_K, SLOTS = [5, 1, 17, 2, 64, 131, 1], [5, 40, 30, 2, 64, 140, 9], [2, 0, 3, 1, 6, 4, 5]


def set_step(n_q, n_k, slots, hints=True):
    ctx, pos = paged_context(n_q, n_k, 8, sum(-(-n // 8) for n in n_k) + 4, 1, DEV, slots=slots)
    if hints:                                           # as the runner gives them; without them every launch is prepared for anything
        ctx.num_leading_decode = next((i for i, n in enumerate(n_q) if n != 1), len(n_q))
        ctx.portion_kinds = nv.ops.portion_kinds(n_q[ctx.num_leading_decode:])
    nv.set_context(ctx)
    return sum(n_q), pos


@pytest.fixture(params=["hints", "no_hints", "singles_first"])
def step(request):
    n_q, n_k = N_Q, N_K
    if request.param == "singles_first":
        order = sorted(range(len(N_Q)), key=lambda i: N_Q[i] != 1)
        n_q, n_k = [N_Q[i] for i in order], [N_K[i] for i in order]
    yield set_step(n_q, n_k, SLOTS, request.param != "no_hints")
    nv.set_context(None)


def rn(g, *s, std=1.0, mean=0.0):
    return (torch.randn(*s, generator=g) * std + mean).to(DEV)


def pair(cls_name, *args, **kw):
    a, b = getattr(hip_layers(), cls_name)(*args, device=DEV, **kw), getattr(R, cls_name)(*args, device=DEV, **kw)
    g = torch.Generator().manual_seed(len(cls_name))
    with torch.no_grad():
        for (_, pa), (_, pb) in zip(a.named_parameters(), b.named_parameters()):
            v = rn(g, *pa.shape, std=0.3, mean=0.2).to(pa.dtype)
            pa.copy_(v), pb.copy_(v)
    for m in (a, b):
        if hasattr(m, "finalize"):
            m.finalize()
    return a, b


@pytest.mark.parametrize("W", [96, 100, 2048, 521])
def test_boundary_with_a_normed_and_scaled_input(dt, W):
    L, g, T = hip_layers(), torch.Generator().manual_seed(W), 9
    norm_a, norm_b = pair("ScaledNorm", W)
    x, y, fw = rn(g, T, W), rn(g, T, W + 3).to(dt)[:, :W], rn(g, W, std=0.2, mean=1.0)
    xa, xb = x.clone(), x.clone()
    a = L.stream_boundary(xa, normed=y, normed_weight=norm_a.applied, eps=1e-6, copy_dtype=dt)
    b = R.stream_boundary(xb, normed=y, normed_weight=norm_b.applied, eps=1e-6, copy_dtype=dt)
    assert rel(xa, xb) < 3e-6 and rel(a, b) < tol(dt)
    a = L.stream_boundary(xa, normed=y, normed_weight=norm_a.applied, norm=fw, eps=1e-6, out_dtype=dt)[1]
    b = R.stream_boundary(xb, normed=y, normed_weight=norm_b.applied, norm=fw, eps=1e-6, out_dtype=dt)[1]
    assert rel(xa, xb) < 3e-6 and rel(a, b) < tol(dt)


@pytest.mark.parametrize("C,N", [(64, 1), (100, 3), (33, 8), (256, 16), (70, 20), (40, 32), (130, 64), (17, 100), (8, 256)])
def test_selective_scan(dt, step, C, N):
    T, _ = step
    a, b = pair("SelectiveScan", C, N)
    g = torch.Generator().manual_seed(C + N)
    R_ = 5
    xz, dbc = rn(g, T, 2 * C).to(dt), rn(g, T, R_ + 2 * N).to(dt)              # slices of wider products
    x, z = xz.split(C, dim=1)
    _, B, Cm = dbc.split((R_, N, N), dim=1)
    raw = rn(g, T, C, std=2.0, mean=-2.0).to(dt)
    sa = rn(g, 8, C, N, std=0.5)
    sb = sa.clone()
    ya, yb = a(x, raw, z, B, Cm, sa), b(x, raw, z, B, Cm, sb)
    assert rel(ya, yb) < tol(dt) and rel(sa[SLOTS], sb[SLOTS]) < 1e-5
    assert torch.equal(sa[7], sb[7])                                           # the slot nobody holds


@pytest.mark.parametrize("C,N,n_q", [(64, 16, [700]), (48, 4, [1, 1111, 300, 2]), (64, 8, [1] * 40 + [900, 3, 1, 650, 17, 1, 800]), (2048, 16, [513]), (2048, 16, [40] * 70)])
def test_selective_scan_segments_and_many_sequences(dt, C, N, n_q):
    """Long portions of few sequences run in segments; many sequences take eight states per lane."""
    slots = list(range(len(n_q)))[::-1]
    T, _ = set_step(n_q, [n + 3 * (i % 2) for i, n in enumerate(n_q)], slots)
    a, b = pair("SelectiveScan", C, N)
    g = torch.Generator().manual_seed(C + len(n_q))
    x, z, B, Cm = rn(g, T, C).to(dt), rn(g, T, C).to(dt), rn(g, T, N).to(dt), rn(g, T, N).to(dt)
    raw = rn(g, T, C, mean=-4.0).to(dt)                                       # small steps: a state outlives several segments
    sa = rn(g, len(n_q), C, N, std=0.5)
    sb = sa.clone()
    ya, yb = a(x, raw, z, B, Cm, sa), b(x, raw, z, B, Cm, sb)
    nv.set_context(None)
    assert rel(ya, yb) < tol(dt) and rel(sa, sb) < 1e-5


@pytest.mark.parametrize("H,G,D,Dv,rot,scaling", [
    (4, 2, 12, 20, 8, {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}), (6, 1, 128, 64, 64, None), (2, 2, 128, 128, 128, None),
    (3, 3, 10, 7, 10, None), (9, 1, 16, 32, 2, None), (2, 1, 160, 96, 32, {"factor": 8.0, "original": 512, "fast": 32.0, "slow": 1.0}),
    (4, 4, 7, 9, 0, None), (64, 4, 256, 16, 96, None)])
def test_row_norm_attention(dt, step, H, G, D, Dv, rot, scaling):
    T, pos = step
    a, b = pair("RowNormAttention", H, G, D, Dv, 1.7 / D ** 0.5, 1e-6, rot, 300.0, scaling)
    g = torch.Generator().manual_seed(H * D)
    with torch.no_grad():
        a.q_norm.add_(1.0), b.q_norm.add_(1.0), a.k_norm.add_(1.0), b.k_norm.add_(1.0)
    n = [H * D, G * D, G * Dv]
    for extra in (3, -sum(n) % 8):                      # rows of a wider product: an odd stride, an aligned one
        qkv = rn(g, T, sum(n) + extra).to(dt)
        q, k, v = qkv[:, :sum(n)].split(n, dim=1)
        q, k, v = q.unflatten(1, (H, D)), k.unflatten(1, (G, D)), v.unflatten(1, (G, Dv))
        nb = sum(-(-x // 8) for x in N_K) + 4
        ka, va = rn(g, nb, 8, G, D).to(dt), rn(g, nb, 8, G, Dv).to(dt)      # stale pages
        kb, vb = ka.clone(), va.clone()
        ya, yb = a(q, k, v, pos, ka, va), b(q, k, v, pos, kb, vb)
        assert rel(ya, yb) < tol(dt) and rel(ka, kb) < tol(dt) and torch.equal(va, vb)


@pytest.mark.parametrize("H,Dk,Dv", [(3, 10, 6), (2, 32, 64), (1, 64, 17), (2, 33, 130), (2, 96, 200), (4, 128, 128), (1, 200, 64), (1, 256, 256)])
def test_fixed_decay_memory(dt, step, H, Dk, Dv):
    T, _ = step
    decay = [0.0, 0.7, 0.999, 1.0][-H:]
    a, b = pair("FixedDecayMemory", H, Dk, Dv, decay)
    g = torch.Generator().manual_seed(Dk)
    n = [H * Dk, H * Dk, H * Dv]
    for extra in (1, -sum(n) % 8):
        qkv = rn(g, T, sum(n) + extra).to(dt)
        q, k, v = qkv[:, :sum(n)].split(n, dim=1)
        q, k, v = q.unflatten(1, (H, Dk)), k.unflatten(1, (H, Dk)), v.unflatten(1, (H, Dv))
        ca = {"state": rn(g, 8, H, Dk, Dv, std=0.5)}
        cb = {"state": ca["state"].clone()}
        ya, yb = a(q, k, v, ca), b(q, k, v, cb)
        # (bf16: the chunks round silu(q), silu(k), silu(v) to bf16 as activations; the stand-in does not)
        assert rel(ya, yb) < tol(dt) and rel(ca["state"][SLOTS], cb["state"][SLOTS]) < (1e-5 if dt == torch.float32 else 5e-3)
        assert torch.equal(ca["state"][7], cb["state"][7])


def test_fixed_decay_chunks_round_nothing_but_the_activations():
    """bfloat16 rows whose SiLU is exact in bfloat16 (0 or a large number): the chunks must then agree with the float32
    recurrence to about 16 bits, although scores, state and values go through bfloat16 operands."""
    H, Dk, Dv, n = 2, 64, 64, 400
    T, _ = set_step([n], [n + 7], [0])
    a, b = pair("FixedDecayMemory", H, Dk, Dv, [0.93, 0.9995])
    g = torch.Generator().manual_seed(3)
    draw = lambda d: torch.where(torch.rand(T, H, d, generator=g) < 0.5, torch.zeros(()), 20.0 + torch.randint(0, 12, (T, H, d), generator=g).float()).to(DEV)
    q, k, v = draw(Dk), draw(Dk), draw(Dv)
    s0 = rn(g, 1, H, Dk, Dv, std=100.0)
    ca, cb = {"state": s0.clone()}, {"state": s0.clone()}
    ya = a(q.bfloat16(), k.bfloat16(), v.bfloat16(), ca)
    yb = b(q, k, v, cb)
    nv.set_context(None)
    assert rel(ya, yb) < 3e-5 and rel(ca["state"], cb["state"]) < 3e-5


@pytest.mark.parametrize("H,Dk,Dv,n_q", [(2, 32, 64, [700]), (1, 64, 32, [1, 1111, 300, 2]), (2, 32, 32, [1] * 40 + [900, 3, 1, 650, 17, 1, 800]), (8, 128, 128, [2048])])
def test_fixed_decay_segments(dt, H, Dk, Dv, n_q):
    slots = list(range(len(n_q)))[::-1]
    T, _ = set_step(n_q, [n + 3 * ((i + 1) % 2) for i, n in enumerate(n_q)], slots)
    a, b = pair("FixedDecayMemory", H, Dk, Dv, [1.0 - 2.0 ** (-4 - h) for h in range(H)])
    g = torch.Generator().manual_seed(Dk)
    q, k, v = rn(g, T, H, Dk).to(dt), rn(g, T, H, Dk).to(dt), rn(g, T, H, Dv).to(dt)
    ca = {"state": rn(g, len(n_q), H, Dk, Dv, std=5.0)}
    cb = {"state": ca["state"].clone()}
    ya, yb = a(q, k, v, ca), b(q, k, v, cb)
    nv.set_context(None)
    assert rel(ya, yb) < tol(dt) and rel(ca["state"], cb["state"]) < (1e-5 if dt == torch.float32 else 5e-3)


@pytest.mark.parametrize("H,Dv,cols", [(4, 16, 64), (3, 7, 45), (16, 128, 2048), (2, 12, 4100), (1, 5, 16384), (5, 8, 1030)])
def test_join_gated(dt, H, Dv, cols):
    T = 7
    a, b = pair("JoinGated", cols, 1e-6, 0.6, 1.9)
    g = torch.Generator().manual_seed(cols)
    z = rn(g, T, cols + H + 5).to(dt)
    attn, mem = rn(g, T, H * Dv).to(dt), rn(g, T, cols, std=30.0)
    ya, yb = a(attn, z[:, cols:cols + H], mem, z[:, :cols]), b(attn, z[:, cols:cols + H], mem, z[:, :cols])
    assert rel(ya[:, :H * Dv], yb[:, :H * Dv]) < tol(dt) and rel(ya[:, H * Dv:], yb[:, H * Dv:]) < tol(dt)


@pytest.mark.parametrize("inter,stride", [(64, 128), (45, 90), (4096, 8192), (20, 43)])
def test_clamped_glu_and_softcap(dt, inter, stride):
    L, g = hip_layers(), torch.Generator().manual_seed(inter)
    x = rn(g, 9, stride, std=3.0).to(dt)[:, :2 * inter]
    assert rel(L.ClampedGLU(1.3)(x), R.ClampedGLU(1.3)(x)) < tol(dt)
    assert rel(L.ClampedGLU(2.0, 1.0, 0.0)(x), R.ClampedGLU(2.0, 1.0, 0.0)(x)) < tol(dt)
    y = x.contiguous()
    assert rel(L.ScaledSoftcap(0.7, 4.0)(y), R.ScaledSoftcap(0.7, 4.0)(y)) < 3e-6
    assert rel(L.ScaledSoftcap(0.7, 0.0)(y), R.ScaledSoftcap(0.7, 0.0)(y)) < 3e-6
