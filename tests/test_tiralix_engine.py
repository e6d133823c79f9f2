"""Tiralix through the engine against the plain oracle (oracle/ref_tiralix.py: whole sequences, no cache).

Every test runs on the CPU with the eager stand-in layers (host logic: scheduler, block and slot managers, runner,
model wiring) and, marked gpu, on the HIP kernels in float32 and bfloat16.  Float32 keeps the comparison tight (a key
that is off by one, a lost state, a stale slot, a gate on the wrong head is far outside it); bfloat16 is bounded per
position by three times the error the oracle's own bfloat16 evaluation makes there.  Small configurations of the tests'
own: odd head counts, key size != value size, partial, full and no rotary, with and without frequency blending, one to
five taps, layers without feed-forward, other head counts on the two sides of a parallel mixer, logits with and without
a cap."""
import pytest
import torch

from nanovllm_amd.engine.sequence import SamplingParams
from oracle import ref_tiralix
from tiralix_util import (config, dense, make_engine, mamba_layer, oracle_logits, parallel_layer, random_checkpoint, rel_err,
                          replay)

BACKENDS = [pytest.param(("cpu", torch.float32), id="cpu-f32"),
            pytest.param(("cuda", torch.float32), id="gpu-f32", marks=pytest.mark.gpu),
            pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=pytest.mark.gpu)]


@pytest.fixture(params=BACKENDS)
def backend(request):
    return request.param


def per_position(got, want):
    d = got.float() - want.float()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.float().pow(2).mean().sqrt()


def assert_close_to_oracle(got, cfg, ck, prompt, dtype, what=""):
    """float32: every position within 5e-5.  bfloat16: against what the oracle's own bfloat16 evaluation loses per position."""
    want = oracle_logits(cfg, ck, prompt, torch.float32)
    assert got.shape == want.shape
    err = per_position(got, want)
    if dtype == torch.float32:
        assert err.max().item() < 5e-5, (what, err.max().item())
        return
    noise = per_position(oracle_logits(cfg, ck, prompt, torch.bfloat16), want)
    limit = 3 * torch.clamp(noise, min=noise.median().item()) + 1e-3
    over = int((err > limit).sum())
    assert over <= max(1, err.numel() // 20), (what, over, (err / limit).topk(min(5, err.numel())).values.tolist())
    assert err.median().item() <= 2 * noise.median().item() + 1e-3, (what, err.median().item(), noise.median().item())


def tokens(n, seed, vocab=91):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


MIXED = config([mamba_layer(), parallel_layer(), parallel_layer(heads=3, kv_heads=1, dim=10, vdim=16, rot_dims=10, scaling=None, rheads=3,
                                                                rdim=16, rvdim=5, left_scale=1.0, right_scale=0.5, mlp=None),
                mamba_layer(inner=23, state=17, dt_rank=1, conv=5, mlp=dense(20, 3.0))])
SINGLE = {"mamba": config([mamba_layer()]),
          "mamba_one_tap_one_state_no_ff": config([mamba_layer(inner=64, state=1, dt_rank=8, conv=1, mlp=None)]),
          "parallel": config([parallel_layer()]),
          "parallel_no_rotary_no_ff": config([parallel_layer(heads=2, kv_heads=2, rot_dims=0, rheads=1, mlp=None)]),
          "parallel_many_query_heads": config([parallel_layer(heads=9, kv_heads=1, dim=8, vdim=8, rot_dims=8, scaling=None)]),
          "no_softcap": config([parallel_layer(), mamba_layer()], logit_scale=1.7, logit_softcap=None)}


def check(engine, cfg, ck, prompts, portions, dtype, order=None):
    got = replay(engine, prompts, portions, order)
    for i, p in prompts.items():
        assert_close_to_oracle(got[i], cfg, ck, p, dtype, i)


@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_layer_kind_alone_whole_prompt_and_token_by_token(backend, name):
    dev, dtype = backend
    cfg = SINGLE[name]
    ck = random_checkpoint(cfg, seed=len(name))
    p = {"a": tokens(41, 1)}
    check(make_engine(cfg, ck, dev, dtype), cfg, ck, p, {"a": [41]}, dtype)
    check(make_engine(cfg, ck, dev, dtype), cfg, ck, p, {"a": [1]}, dtype)


def test_whole_model_portions_of_many_sizes(backend):
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=2)
    p = {"a": tokens(75, 3)}
    for sizes in ([75], [2], [3, 2, 7, 1, 1, 16, 2, 5], [17, 16, 18], [1, 4, 4, 4], [64, 1], [6, 1, 7, 7]):
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
    want_logits, want = ref_tiralix.forward(MIXED, ck, toks, dtype)
    assert len(streams) == want.shape[0] == 4
    for r, s in enumerate(streams):
        torch.testing.assert_close(s.cpu(), want[r], rtol=1e-4, atol=1e-4)
    assert rel_err(got.cpu(), want_logits[[0, 18]]) < 5e-5


def test_unequal_requests_in_one_batch_equal_each_alone(backend):
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=6)
    p = {"a": tokens(60, 7), "b": tokens(9, 8), "c": tokens(1, 9), "d": tokens(43, 10)}
    portions = {"a": [5, 1, 1, 29, 1], "b": [1], "c": [1], "d": [2, 31, 1]}
    eng = make_engine(MIXED, ck, dev, dtype)
    check(eng, MIXED, ck, p, portions, dtype, order={"b": 1, "d": 2})
    if dtype != torch.float32:
        return
    together = replay(make_engine(MIXED, ck, dev, dtype), p, portions, order={"b": 1, "d": 2})
    for i in p:
        alone = replay(make_engine(MIXED, ck, dev, dtype), {i: p[i]}, {i: portions[i]})
        assert rel_err(together[i], alone[i]) < 5e-5


def test_pages_and_slots_are_used_again(backend):
    """A pool that holds two requests at a time, six requests in a row: every page and both slots are reused with
    what the previous owner left in them (keys and values, both kinds of state, carried convolution inputs)."""
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=11)
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=15, max_seqs=2)
    for r in range(3):
        p = {f"x{r}": tokens(31 - r, 20 + r), f"y{r}": tokens(13 + 3 * r, 30 + r)}
        got = replay(eng, p, {f"x{r}": [20, 2, 1], f"y{r}": [1, 5]})
        for i in p:
            assert_close_to_oracle(got[i], MIXED, ck, p[i], dtype, (r, i))
        assert eng.scheduler.block_manager.num_free_blocks == 15 and eng.scheduler.state_slots.num_free == 2
    assert not eng.scheduler.running and not eng.scheduler.waiting
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=3, max_seqs=1)
    eng.replay_step([("a", tokens(5, 1), [])])
    with pytest.raises(ValueError):
        eng.replay_step([("b", tokens(2, 2), [])])
    with pytest.raises(ValueError):
        eng.replay_step([("a", tokens(9, 3), [])])


def test_a_request_left_out_of_steps_goes_on_from_its_own_state(backend):
    dev, dtype = backend
    ck = random_checkpoint(MIXED, seed=26)
    a, b = tokens(50, 27), tokens(37, 28)
    eng = make_engine(MIXED, ck, dev, dtype, num_blocks=24, max_seqs=2)
    rows = lambda n: list(range(n))
    got_a = [eng.replay_step([("a", a[:18], rows(18))]).cpu()]
    got_b = [eng.replay_step([("b", b[:20], rows(20))]).cpu()]
    for t in range(20, 24):
        got_b.append(eng.replay_step([("b", b[t:t + 1], [0])]).cpu())
    both = eng.replay_step([("b", b[24:], rows(13)), ("a", a[18:], rows(32))], ["a", "b"]).cpu()
    assert_close_to_oracle(torch.cat(got_a + [both[13:]]), MIXED, ck, a, dtype, "a")
    assert_close_to_oracle(torch.cat(got_b + [both[:13]]), MIXED, ck, b, dtype, "b")


def test_long_decoding_past_every_edge(backend):
    """A short prompt and 140 single tokens: they cross page borders (every 4) and the blended rotary band and leave the
    first tokens far behind, reachable through the attention's cache and both recurrent states."""
    dev, dtype = backend
    cfg = config([parallel_layer(decay=[0.3, 0.9995]), mamba_layer(mlp=dense())])
    ck = random_checkpoint(cfg, seed=12)
    p = {"a": tokens(143, 13)}
    check(make_engine(cfg, ck, dev, dtype, num_blocks=40), cfg, ck, p, {"a": [3, 1]}, dtype)


def test_greedy_generation_through_generate(backend):
    dev, dtype = backend
    if dtype != torch.float32:
        pytest.skip("token equality is asserted in float32")
    ck = random_checkpoint(MIXED, seed=14)
    prompts = [tokens(11, 15), tokens(3, 16), tokens(26, 17)]
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=40, max_seqs=2,       # the third waits for a slot
                      max_num_batched_tokens=16, long_prefill_token_threshold=6)
    outs, _ = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10))
    for p, o in zip(prompts, outs):
        seq = list(p)
        for _ in range(10):
            seq.append(int(oracle_logits(MIXED, ck, seq, dtype)[-1].argmax()))
        assert o["token_ids"] == seq[len(p):]
    assert eng.scheduler.state_slots.num_free == 2 and eng.scheduler.block_manager.num_free_blocks == 40


def test_preemption_recomputes_state_and_sampling_runs(backend):
    dev, dtype = backend
    if dtype != torch.float32:
        pytest.skip("token equality is asserted in float32")
    ck = random_checkpoint(MIXED, seed=18)
    prompts = [tokens(10, 19), tokens(9, 20)]
    eng = make_engine(MIXED, ck, dev, dtype, block_size=4, num_blocks=9, max_seqs=2)
    outs, _ = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert sum(o["num_preemptions"] for o in outs) >= 1
    for p, o in zip(prompts, outs):
        seq = list(p)
        for _ in range(12):
            seq.append(int(oracle_logits(MIXED, ck, seq, dtype)[-1].argmax()))
        assert o["token_ids"] == seq[len(p):]
    outs, _ = make_engine(MIXED, ck, dev, dtype).generate(prompts, SamplingParams(temperature=0.8, max_tokens=5))
    assert all(len(o["token_ids"]) == 5 for o in outs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_sizes_of_the_matrix_core_kernels_through_the_engine(dtype):
    """Key sizes 64 and 128: prompt portions of the attention take its tile kernel, single rows its decode kernel, portions of
    more than 16 tokens of the linear attention its chunks (key sizes 96 and 128, value sizes that are and are not whole
    groups of 64 columns), the scan 4 to 16 lanes per channel; pages of 16."""
    cfg = config([parallel_layer(heads=12, kv_heads=2, dim=64, vdim=32, rot_dims=32, rheads=3, rdim=96, rvdim=72, mlp=dense(64)),
                  mamba_layer(inner=160, state=64, dt_rank=12, conv=4, mlp=None),
                  parallel_layer(heads=4, kv_heads=2, dim=128, vdim=128, rot_dims=128, rheads=2, rdim=128, rvdim=128, mlp=dense(40)),
                  mamba_layer(inner=96, state=16, dt_rank=6, conv=2)], width=64)
    ck = random_checkpoint(cfg, seed=21)
    p = {"a": tokens(333, 22), "b": tokens(70, 23), "c": tokens(150, 24)}
    eng = make_engine(cfg, ck, "cuda", dtype, block_size=16, num_blocks=64)
    check(eng, cfg, ck, p, {"a": [130, 1, 67, 64, 1, 70], "b": [1], "c": [65, 2, 83]}, dtype, order={"b": 1, "c": 2})


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_the_largest_sizes_through_the_engine(dtype):
    """Memories of up to 256 x 256 channels (token by token: the chunks are built for keys of at most 128), attention heads of
    160 and 256 dimensions, 256 states per channel (all 64 lanes of a wave), eleven taps (beyond the register window)."""
    cfg = config([parallel_layer(heads=2, kv_heads=1, dim=160, vdim=256, rot_dims=64, rheads=1, rdim=200, rvdim=160, mlp=None),
                  mamba_layer(inner=30, state=256, dt_rank=3, conv=11, mlp=dense(96)),
                  parallel_layer(heads=2, kv_heads=2, dim=256, vdim=48, rot_dims=256, scaling=None, rheads=1, rdim=256, rvdim=256),
                  mamba_layer(inner=33, state=100, dt_rank=40, conv=2, mlp=None)], width=48)
    ck = random_checkpoint(cfg, seed=41)
    p = {"a": tokens(150, 42), "b": tokens(40, 43)}
    eng = make_engine(cfg, ck, "cuda", dtype, block_size=16, num_blocks=24)
    check(eng, cfg, ck, p, {"a": [70, 1, 2, 66, 1], "b": [1]}, dtype, order={"b": 1})


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])
def test_long_prompts_are_cut_into_segments_along_time(dtype):
    """Prompts long enough for both recurrences to run in segments (at least 512 tokens and few sequences), continued from a
    carried state, beside shorter portions and single tokens."""
    cfg = config([mamba_layer(inner=48, state=8, mlp=None), parallel_layer(heads=2, kv_heads=1, dim=16, vdim=16, rot_dims=16, rheads=2,
                                                                           rdim=32, rvdim=64, decay=[0.9, 0.9993], mlp=None)], width=40)
    ck = random_checkpoint(cfg, seed=51)
    p = {"a": tokens(1330, 52), "b": tokens(37, 53), "c": tokens(700, 54)}
    eng = make_engine(cfg, ck, "cuda", dtype, block_size=16, num_blocks=140)
    check(eng, cfg, ck, p, {"a": [600, 1, 729], "b": [1, 30, 1], "c": [3, 1, 696]}, dtype, order={"b": 0, "c": 0})
