"""Nekodra through the engine against the plain oracle (oracle/ref_nekodra.py: whole sequences, no cache).

Every test runs on the CPU with the eager stand-in layers (host logic: scheduler, block manager, runner, model wiring) and,
marked gpu, on the HIP kernels in float32 and bfloat16.  Float32 keeps the comparison tight (a key that is off by one, a
stale page, a missing sink or a wrong expert is far outside it); bfloat16 is bounded by three times the error the oracle's
own bfloat16 evaluation makes.  Small configurations of the tests' own: odd head counts, one head, key size != value size
!= latent size, latents shared by none, one and several later layers that are not neighbours, layers of unequal sizes,
with and without identity experts, shared expert and feed-forward, top 1 and top = all."""
import pytest
import torch

from nanovllm_amd.engine.sequence import SamplingParams
from oracle import ref_nekodra
from nekodra_util import assert_close_to_oracle, config, layer, make_engine, moe, oracle_logits, random_checkpoint, rel_err, replay

BACKENDS = [pytest.param(("cpu", torch.float32), id="cpu-f32"),
            pytest.param(("cuda", torch.float32), id="gpu-f32", marks=pytest.mark.gpu),
            pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=pytest.mark.gpu)]


@pytest.fixture(params=BACKENDS)
def backend(request):
    return request.param


def tokens(n, seed, vocab=83):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


# two latent caches, read by layers 0, 2, 4 and by layers 1, 5; layer 3 has its own and no feed-forward
MIXED = config([layer(), layer(heads=2, dim=16, vdim=8, rank=24, mlp=moe(experts=4, identity=0, top=1, shared=0)),
                layer(heads=5, dim=6, vdim=9, kv_from=0, mlp=moe(experts=3, identity=3, top=6, scale=0.8)),
                layer(heads=1, dim=7, vdim=21, rank=33, mlp=None), layer(kv_from=0, mlp=moe(experts=9, identity=1, top=2, shared=0)),
                layer(heads=4, dim=12, vdim=12, rank=24, kv_from=1)])
SINGLE = {"own_latent": config([layer()]), "no_ff": config([layer(heads=1, mlp=None)]),
          "one_expert_all_identity_choices": config([layer(mlp=moe(experts=1, identity=5, top=4))]),
          "no_identity_no_shared": config([layer(heads=7, dim=3, vdim=2, rank=5, mlp=moe(identity=0, shared=0))]),
          "sizes_alike": config([layer(heads=4, dim=16, vdim=16, rank=16)]), "shared_latent": config([layer(), layer(heads=6, kv_from=0)])}


def check(engine, cfg, ck, prompts, portions, dtype, order=None):
    got = replay(engine, prompts, portions, order)
    for i, p in prompts.items():
        assert_close_to_oracle(got[i], cfg, ck, p, dtype, i)


@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_kind_of_layer_alone_whole_prompt_and_token_by_token(backend, name):
    dev, dtype = backend
    cfg = SINGLE[name]
    ck = random_checkpoint(cfg, seed=len(name))
    p = {"a": tokens(41, 1)}
    check(make_engine(cfg, ck, dev, dtype), cfg, ck, p, {"a": [41]}, dtype)
    check(make_engine(cfg, ck, dev, dtype), cfg, ck, p, {"a": [1]}, dtype)


def test_whole_model_portions_of_many_sizes(backend):
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=2)
    p = {"a": tokens(53, 3)}
    for sizes in ([53], [2], [3, 2, 7, 1, 1, 16, 2, 5], [1, 4, 4, 4], [17, 1], [6, 1, 7, 7]):
        check(make_engine(MIXED, ck, dev, dtype), MIXED, ck, p, {"a": sizes}, dtype)


def test_streams_after_every_layer_match_the_oracle(backend):
    dev, dtype = backend
    if dtype != torch.float32:
        pytest.skip("streams are compared in float32")
    ck = random_checkpoint(MIXED, seed=4)
    toks = tokens(19, 5)
    eng = make_engine(MIXED, ck, dev, dtype)
    streams = []
    model = eng.runner.model
    orig = model.forward
    model.forward = lambda *a, **k: orig(*a, streams=streams, **k)
    got = eng.replay_step([("a", toks, [0, 18])], ["a"])
    want_logits, want = ref_nekodra.forward(MIXED, ck, toks, dtype)
    assert len(streams) == want.shape[0] == 6
    for s, w in zip(streams, want):
        torch.testing.assert_close(s.cpu(), w, rtol=1e-4, atol=1e-4)
    assert rel_err(got.cpu(), want_logits[[0, 18]]) < 5e-5


def test_unequal_requests_in_one_batch_equal_each_alone(backend):
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=6)
    p = {"a": tokens(37, 7), "b": tokens(9, 8), "c": tokens(1, 9), "d": tokens(23, 10)}
    portions = {"a": [5, 1, 1, 9, 1], "b": [1], "c": [1], "d": [2, 11, 1]}
    check(make_engine(MIXED, ck, dev, dtype), MIXED, ck, p, portions, dtype, order={"b": 1, "d": 2})
    if dtype != torch.float32:
        return
    together = replay(make_engine(MIXED, ck, dev, dtype), p, portions, order={"b": 1, "d": 2})
    for i in p:
        alone = replay(make_engine(MIXED, ck, dev, dtype), {i: p[i]}, {i: portions[i]})
        assert rel_err(together[i], alone[i]) < 5e-5


def test_pages_are_used_again(backend):
    """A pool that holds two requests at a time, six requests in a row: every page is reused with the latents that the
    previous owner left in it; a request too many, too long or beyond the position table is refused."""
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=11)
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=12, max_seqs=2)
    for r in range(3):
        p = {f"x{r}": tokens(22 - r, 20 + r), f"y{r}": tokens(13 + 3 * r, 30 + r)}
        got = replay(eng, p, {f"x{r}": [7, 2, 1], f"y{r}": [1, 5]})
        for i in p:
            assert_close_to_oracle(got[i], MIXED, ck, p[i], dtype, (r, i))
        assert eng.scheduler.block_manager.num_free_blocks == 12
    assert not eng.scheduler.running and not eng.scheduler.waiting
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=3, max_seqs=1)
    eng.replay_step([("a", tokens(5, 1), [])])
    with pytest.raises(ValueError):
        eng.replay_step([("a", tokens(9, 3), [])])
    eng = make_engine({**MIXED, "max_positions": 12}, {**ck, "pos": ck["pos"][:12]}, dev, dtype)
    eng.replay_step([("a", tokens(10, 1), [])])
    with pytest.raises(ValueError):
        eng.replay_step([("a", tokens(3, 3), [])])
    got = eng.replay_step([("a", tokens(2, 3), [1])])
    assert rel_err(got.cpu(), oracle_logits(MIXED, ck, tokens(10, 1) + tokens(2, 3), torch.float32)[[11]]) < (5e-5 if dtype == torch.float32 else 6e-2)
    with pytest.raises(ValueError):
        eng.add_request(tokens(10, 1), SamplingParams(temperature=0.0, max_tokens=3))


def test_long_decoding(backend):
    """A short prompt and 140 single tokens: they cross page borders (every 4) and leave the first tokens far behind."""
    dev, dtype = backend
    cfg = config([layer(), layer(heads=2, kv_from=0), layer(rank=20)])
    ck = random_checkpoint(cfg, seed=12)
    p = {"a": tokens(143, 13)}
    check(make_engine(cfg, ck, dev, dtype, num_blocks=40), cfg, ck, p, {"a": [3, 1]}, dtype)


def greedy(cfg, ck, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(oracle_logits(cfg, ck, seq)[-1].argmax()))
    return seq[len(prompt):]


def test_greedy_generation_through_generate(backend):
    dev, dtype = backend
    if dtype != torch.float32:
        pytest.skip("token equality is asserted in float32")
    ck = random_checkpoint(MIXED, seed=14)
    prompts = [tokens(11, 15), tokens(3, 16), tokens(26, 17)]
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=40, max_seqs=2,       # the third waits
                      max_num_batched_tokens=16, long_prefill_token_threshold=6)
    outs, _ = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10))
    for p, o in zip(prompts, outs):
        assert o["token_ids"] == greedy(MIXED, ck, p, 10)
    assert eng.scheduler.block_manager.num_free_blocks == 40


def test_a_cached_prefix_is_taken_over(backend):
    """Everything a sequence leaves behind is in its pages: a second prompt with the same first tokens starts from them."""
    dev, dtype = backend
    if dtype != torch.float32:
        pytest.skip("token equality is asserted in float32")
    ck = random_checkpoint(MIXED, seed=15)
    head = tokens(18, 25)
    first, second = head + tokens(5, 26), head + tokens(7, 27)
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=40)
    eng.generate([first], SamplingParams(temperature=0.0, max_tokens=2))
    outs, _ = eng.generate([second], SamplingParams(temperature=0.0, max_tokens=8))
    assert outs[0]["cached_tokens"] == 16
    assert outs[0]["token_ids"] == greedy(MIXED, ck, second, 8)


def test_preemption_recomputes_and_sampling_runs(backend):
    dev, dtype = backend
    if dtype != torch.float32:
        pytest.skip("token equality is asserted in float32")
    ck = random_checkpoint(MIXED, seed=18)
    prompts = [tokens(10, 19), tokens(9, 20)]
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=9, max_seqs=2)
    outs, _ = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert sum(o["num_preemptions"] for o in outs) >= 1
    for p, o in zip(prompts, outs):
        assert o["token_ids"] == greedy(MIXED, ck, p, 12)
    outs, _ = make_engine(MIXED, ck, dev, dtype).generate(prompts, SamplingParams(temperature=0.8, max_tokens=5))
    assert all(len(o["token_ids"]) == 5 for o in outs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_sizes_of_the_matrix_core_kernels_through_the_engine(dtype):
    """Latents of 64, 128 and 160 columns with 12, 16 and 3 heads, experts wide enough for several column tiles; prompt
    portions beside single rows, pages of 16."""
    cfg = config([layer(heads=12, dim=64, vdim=32, rank=64, mlp=moe(experts=9, identity=2, top=3, ff=72, shared=136)),
                  layer(heads=16, dim=32, vdim=48, rank=128, mlp=None), layer(heads=3, dim=48, vdim=64, rank=160, mlp=moe(ff=64)),
                  layer(heads=20, dim=24, vdim=16, rank=128, kv_from=1)], width=64, positions=400)
    ck = random_checkpoint(cfg, seed=21)
    p = {"a": tokens(333, 22), "b": tokens(70, 23), "c": tokens(150, 24)}
    eng = make_engine(cfg, ck, "cuda", dtype, block_size=16, num_blocks=64)
    check(eng, cfg, ck, p, {"a": [130, 1, 67, 64, 1, 70], "b": [1], "c": [65, 2, 83]}, dtype, order={"b": 1, "c": 2})


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_the_largest_latents_through_the_engine(dtype):
    cfg = config([layer(heads=5, dim=40, vdim=24, rank=256, mlp=None), layer(heads=2, dim=64, vdim=64, rank=512, mlp=moe(experts=3, ff=40)),
                  layer(heads=33, dim=8, vdim=8, rank=256, kv_from=0, mlp=None)], width=48, positions=200)
    ck = random_checkpoint(cfg, seed=41)
    p = {"a": tokens(150, 42), "b": tokens(40, 43)}
    eng = make_engine(cfg, ck, "cuda", dtype, block_size=16, num_blocks=24)
    check(eng, cfg, ck, p, {"a": [70, 1, 2, 66, 1], "b": [1]}, dtype, order={"b": 1})
