"""Each Nekodra mechanism alone, against the plain functions of oracle/ref_nekodra.py, on inputs made so that a fault shows:
the model's own modules (built on the eager stand-in layers on the CPU and, marked gpu, on the HIP kernels in float32) are
driven step by step through a paged cache with stale pages, and compared with the oracle's whole-sequence result.

  * embedding: the position's row, counted from the start of the sequence and not of the portion;
  * attention: a peaked softmax so that one missing or misplaced key moves the output; one key far back, or at a page's
    edge, that a query is aimed at, in prompts and in decoding; the key just ahead of the query made to stand out (it must
    weigh nothing); sinks that take nearly everything, nearly nothing, and that must not be scaled; a gate that reads
    the mixer's input; latents of an earlier layer behind queries of one's own; a latent norm with an eps that matters;
  * routing: corrections that turn the choice but not the weights; identity experts; top of one and of all;
  * the boundary: both norms of the same row, before and after the parts are added."""
import math

import pytest
import torch

from nanovllm_amd.model import nekodra as M
from nekodra_util import layer, layer_namespace, moe
from oracle import ref_nekodra as O
from test_divadra_mechanisms import close, rn, run_in_steps

BACKENDS = [pytest.param("cpu", id="cpu"), pytest.param("cuda", id="gpu", marks=pytest.mark.gpu)]
F32 = torch.float32


@pytest.fixture(params=BACKENDS)
def dev(request):
    return request.param


def lin(g, o, i, gain=1.0):
    return rn(g, o, i, std=gain / math.sqrt(i))


def load(module, w, **place_kw):
    params, seen = dict(module.named_parameters()), set()

    def take(name):
        seen.add(name)
        return w[name]
    with torch.no_grad():
        module.place("", take, **place_kw)
        for ck, pn in module.names("", "").items():
            params[pn].copy_(take(ck))
    assert seen == set(w), set(w) ^ seen
    module.finalize()


def mixer(dev, W, w, eps=1e-5, **sizes):
    L = layer(**sizes)
    cfg = {"vocab": 4, "width": W, "max_positions": 8, "norm": {"eps": eps},
           "layers": [layer(rank=L["mixer"]["kv_rank"], mlp=None), dict(L, mlp=None)]}
    mod = M.NekodraAttention(M.NekodraConfig.from_dict(cfg).layers[1].mixer, W, eps, layer_namespace(dev), F32, dev)
    load(mod, w)
    return mod, L["mixer"]


def weights(g, W, heads, dim, vdim, rank, own=True, gain=1.0):
    w = {"q": lin(g, heads * dim, W, gain), "g": lin(g, heads * vdim, W, 2.0), "o": lin(g, W, heads * vdim),
         "uk": lin(g, heads * dim, rank), "uv": lin(g, heads * vdim, rank), "sink": rn(g, heads)}
    if own:
        w["dkv"], w["dkv.norm"] = lin(g, rank, W), rn(g, rank, std=0.4, mean=1.0)
    return w


def cache(dev, nb, rank, bs=4):
    kc = torch.randn(nb, bs, 1, rank, device=dev)                          # stale pages
    return kc, kc[..., :rank]


def expected(m, w, h, eps=1e-5, c=None):
    return O.latent_attention(m, w, "", h, c if c is not None else O.latents(w, "", h, eps, F32), F32)


# ------------------------------------------------------------------------------------------------ embedding
def test_embedding_adds_the_row_of_the_position(dev):
    g = torch.Generator().manual_seed(1)
    V, W, P = 50, 24, 40
    w = {"embed": rn(g, V, W), "pos": rn(g, P, W, std=3.0)}
    emb = layer_namespace(dev).PositionEmbedding(V, P, W, dtype=F32, device=dev)
    with torch.no_grad():
        emb.weight.copy_(w["embed"]), emb.pos.copy_(w["pos"])
    toks, other = torch.randint(0, V, (P,), generator=g), torch.randint(0, V, (9,), generator=g)
    for portions in ([P], [1], [7, 1, 2, 1]):
        close(run_in_steps(emb, toks, portions, dev, other=other), O.embed(w, toks.tolist()), 1e-6)


# ------------------------------------------------------------------------------------------------ attention
@pytest.mark.parametrize("heads,dim,vdim,rank", [(4, 8, 6, 20), (1, 5, 16, 7), (9, 16, 3, 32), (3, 33, 20, 64), (2, 4, 4, 4), (18, 8, 8, 16)])
def test_attention_peaked_softmax_every_key_counts(dev, heads, dim, vdim, rank):
    g = torch.Generator().manual_seed(heads)
    W, T = 24, 150
    w = weights(g, W, heads, dim, vdim, rank)
    mod, m = mixer(dev, W, w, heads=heads, dim=dim, vdim=vdim, rank=rank, scale=5.0 / math.sqrt(dim))
    h, other = rn(g, T, W), rn(g, 12, W)
    want = expected(m, w, h)
    for portions in ([T], [1], [2, 3, 1, 1, 64, 2, 70], [5, 3]):
        kv = cache(dev, 80, rank)
        close(run_in_steps(lambda x, pos: mod(x, kv), h, portions, dev, other=other), want)


@pytest.mark.parametrize("target,query,portions", [(0, 299, [1]), (3, 299, [296, 1]), (4, 298, [300]), (131, 260, [128, 4, 1]), (63, 64, [64, 2]),
                                                    (64, 300, [65, 1]), (299, 299, [7, 1]), (256, 257, [256, 2]), (200, 199, [300]), (200, 199, [200, 1])])
def test_attention_one_key_stands_out(dev, target, query, portions):
    """Input rows are [query part | latent part]: the query's score with the target is large and every other one is moderate.
    The output of head 0 is then the target's value; a target just ahead of the query weighs nothing."""
    g = torch.Generator().manual_seed(5)
    heads, D, Dv, rank, T = 2, 8, 8, 8, 301
    W = heads * D + rank
    eye = torch.eye(W)
    w = {"q": eye[:heads * D], "dkv": eye[heads * D:], "dkv.norm": torch.ones(rank), "sink": torch.tensor([-2.0, 1.0]),
         "uk": torch.eye(D).repeat(heads, 1), "uv": rn(g, heads * Dv, rank), "g": torch.zeros(heads * Dv, W), "o": rn(g, W, heads * Dv)}
    w["o"][:, Dv:] = 0.0                                                  # only head 0 is looked at
    mod, m = mixer(dev, W, w, heads=heads, dim=D, vdim=Dv, rank=rank, scale=6.0)
    aim = torch.tensor([1.0, -1.0, 1.0, 1.0, -1.0, 1.0, 1.0, -1.0])
    away = torch.tensor([1.0, 1.0, 1.0, -1.0, 1.0, 1.0, -1.0, -1.0])       # orthogonal to aim
    h = rn(g, T, W, std=0.3)
    h[:, heads * D:] += 3.0 * away
    h[target, heads * D:] = 3.0 * aim
    h[query, :D] = aim
    want = expected(m, w, h)
    value = 0.5 * w["uv"][:Dv] @ (aim / math.sqrt(1 + 1e-5 / 9))            # the gate of zeros is sigmoid(0)
    alone = O.linear(torch.cat([value, torch.zeros(Dv)]), w["o"])
    near = (want[query] - alone).norm() < 0.05 * alone.norm()
    assert bool(near) == (target <= query)
    kv = cache(dev, 160, rank)
    close(run_in_steps(lambda x, pos: mod(x, kv), h, portions, dev, num_blocks=160, other=rn(g, 5, W)), want)


def test_the_sink_counts_once_unscaled_and_has_no_value(dev):
    """Score scale 0.01: every score is about 0, so a sink of ln(n) takes the weight of n keys; scaled, left out or given a
    value it would not.  Seen by the first tokens most of all, whose few keys it drowns."""
    g = torch.Generator().manual_seed(6)
    W, T, heads, dim, vdim, rank = 16, 90, 3, 8, 4, 12
    w = weights(g, W, heads, dim, vdim, rank)
    w["sink"] = torch.tensor([math.log(30.0), -40.0, 4.0])
    mod, m = mixer(dev, W, w, heads=heads, dim=dim, vdim=vdim, rank=rank, scale=0.01)
    h = rn(g, T, W)
    want = expected(m, w, h)
    scaled = expected(m, dict(w, sink=w["sink"] * 0.01), h)
    none = expected(m, dict(w, sink=torch.full((heads,), -1e4)), h)
    for wrong in (scaled, none):
        assert (want[0] - wrong[0]).norm() > 0.3 * wrong[0].norm() and (want - wrong).norm() > 0.1 * want.norm()
    for portions in ([T], [1], [2, 1, 30, 2]):
        kv = cache(dev, 80, rank)
        close(run_in_steps(lambda x, pos: mod(x, kv), h, portions, dev, other=rn(g, 7, W)), want)
    w["sink"] = torch.tensor([60.0, 95.0, -80.0])                          # far beyond every score: no overflow, nearly no output
    mod, m = mixer(dev, W, w, heads=heads, dim=dim, vdim=vdim, rank=rank, scale=0.01)
    kv = cache(dev, 80, rank)
    got = run_in_steps(lambda x, pos: mod(x, kv), h, [31, 1, 2], dev)
    assert torch.isfinite(got).all()
    close(got, expected(m, w, h))


def test_latents_of_another_layer_behind_own_queries(dev):
    """The sharing layer reads the other layer's cached rows (as its norm left them) with its own queries, up-projections,
    sink, gate and sizes, and writes nothing into them."""
    g = torch.Generator().manual_seed(8)
    W, T, rank = 20, 70, 24
    wa, wb = weights(g, W, 3, 8, 6, rank), weights(g, W, 5, 4, 9, rank, own=False, gain=3.0)
    a, ma = mixer(dev, W, wa, heads=3, dim=8, vdim=6, rank=rank)
    b, mb = mixer(dev, W, wb, heads=5, dim=4, vdim=9, rank=rank, kv_from=0, scale=1.5)
    assert b.attn.latent_norm is None and not hasattr(b, "dkv")
    ha, hb = rn(g, T, W), rn(g, T, W)
    want = expected(mb, wb, hb, c=O.latents(wa, "", ha, 1e-5, F32))
    for portions in ([T], [1], [2, 33, 1]):
        kv = cache(dev, 80, rank)

        def step(x, pos):
            a(x[:, :W].contiguous(), kv)
            before = kv[0].clone()
            y = b(x[:, W:].contiguous(), kv)
            assert torch.equal(before, kv[0])
            return y
        close(run_in_steps(step, torch.cat([ha, hb], dim=1), portions, dev, other=rn(g, 5, 2 * W)), want)


def test_latent_norm_has_its_eps_inside_the_root_and_the_gate_reads_the_input(dev):
    g = torch.Generator().manual_seed(9)
    W, T, eps = 16, 30, 0.05
    w = weights(g, W, 2, 6, 5, 10)
    mod, m = mixer(dev, W, w, eps=eps, heads=2, dim=6, vdim=5, rank=10)
    h = rn(g, T, W, std=0.2)
    want = expected(m, w, h, eps)
    assert (want - expected(m, w, h, 1e-6)).norm() > 0.1 * want.norm()
    kv = cache(dev, 80, 10)
    close(run_in_steps(lambda x, pos: mod(x, kv), h, [4, 1], dev), want)


# ------------------------------------------------------------------------------------------------ feed-forward, boundary
def ff_module(dev, g, W, c):
    E, n = c["router"]["experts"], c["router"]["experts"] + c["router"]["identity"]
    w = {"router": rn(g, n, W, std=0.5)}
    units = [(f"e{e}.", c["expert"]["ff"]) for e in range(E)] + ([("shared.", c["shared"]["ff"])] if "shared" in c else [])
    for u, ff in units:
        w[u + "gate"], w[u + "up"], w[u + "down"] = lin(g, ff, W, 2.0), lin(g, ff, W, 2.0), lin(g, W, ff)
    w["correction"] = rn(g, n, std=0.15)
    cfg = M.NekodraConfig.from_dict({"vocab": 4, "width": W, "max_positions": 8, "norm": {"eps": 1e-5}, "layers": [layer(mlp=c)]})
    mod = M.NekodraMoE(cfg.layers[0].mlp, W, layer_namespace(dev), F32, dev)
    with torch.no_grad():
        mod.router_weight.copy_(w["router"])
        mod.place("", w.__getitem__, w.__contains__)
    return mod, w


@pytest.mark.parametrize("c", [moe(experts=6, identity=3, top=4), moe(experts=1, identity=0, top=1, shared=0), moe(experts=2, identity=6, top=8, scale=0.5),
                               moe(experts=70, identity=5, top=7, ff=9), moe(experts=5, identity=2, top=1, scale=1.0, shared=0)], ids=str)
def test_routed_experts_identity_experts_and_shared_expert(dev, c):
    L, g = layer_namespace(dev), torch.Generator().manual_seed(c["router"]["experts"])
    W, T = 20, 45
    mod, w = ff_module(dev, g, W, c)
    h = rn(g, T, W)
    h[3] = 12.0 * w["router"][-1] / w["router"][-1].norm()                 # the last expert's score is nearly 1
    ids, wts = O.route(c, w, "", h)
    plain_ids, _ = O.route(c, {k: v for k, v in w.items() if k != "correction"}, "", h)
    if c["router"]["top"] < c["router"]["experts"]:
        assert (ids.sort(1).values != plain_ids.sort(1).values).any()      # the correction turns choices ...
    s = torch.softmax(h @ w["router"].t(), dim=-1)
    close(wts, s.gather(1, ids) * c["router"]["scale"], 1e-6)              # ... and not weights
    got_ids, got_w = mod.router((h @ w["router"].t()).to(dev))
    assert got_ids.cpu().sort(1).values.tolist() == ids.sort(1).values.tolist()
    close(got_w.cpu().sort(1).values, wts.sort(1).values, 1e-5)
    x = rn(g, T, W)
    want = x + O.moe(c, w, "", h, F32)
    shared, routed = mod(h.to(dev), None)
    xd = x.clone().to(dev)
    L.layernorm_pair_boundary(xd, adds=shared, routed=routed)
    close(xd.cpu(), want)


def test_boundary_reads_one_row_through_both_norms(dev):
    L, g = layer_namespace(dev), torch.Generator().manual_seed(15)
    T, W, n = 11, 28, 3
    x, a1, a2, through = rn(g, T, W, mean=4.0), rn(g, T, W), rn(g, T, W), rn(g, T, W)
    parts, wts = rn(g, T, n, W), torch.rand(T, n, generator=g)
    ids = torch.tensor([[0, 1, 5], [5, 6, 2], [4, 5, 6]] * 4)[:T].to(torch.int32)
    wa, ba, wb, bb = rn(g, W, mean=1.0), rn(g, W), rn(g, W, mean=1.0), rn(g, W)
    to = lambda t: t.to(dev)
    xd = to(x.clone())
    pair = lambda **kw: L.layernorm_pair_boundary(xd, norm_a=(to(wa), to(ba)), norm_b=(to(wb), to(bb)), eps=1e-3, out_dtype=F32, want_f32_b=True, **kw)
    h1, h2, h32 = pair()                                                  # the first norms: nothing is added
    close(h1.cpu(), O.layer_norm(x, wa, ba, 1e-3), 1e-6), close(h2.cpu(), O.layer_norm(x, wb, bb, 1e-3), 1e-6)
    h1, h2, h32 = pair(adds=[to(a1), to(a2)], routed=(to(parts), to(ids), to(wts), 5, to(through)))
    product = (ids < 5)[:, :, None]
    want = x + a1 + a2 + torch.where(product, parts, wts[:, :, None] * through[:, None]).sum(1)
    close(xd.cpu(), want, 1e-6)
    close(h1.cpu(), O.layer_norm(want, wa, ba, 1e-3), 1e-6), close(h2.cpu(), O.layer_norm(want, wb, bb, 1e-3), 1e-6)
    assert torch.equal(h2, h32)
    L.layernorm_pair_boundary(xd, adds=[to(a1)])                          # no norm
    close(xd.cpu(), want + a1, 1e-6)
