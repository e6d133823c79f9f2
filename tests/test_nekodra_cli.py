"""Nekodra from a checkpoint directory: config.json -> registry -> model, *.safetensors -> parameters, and the two
command-line programs.  CPU: the registry and loader with the eager stand-in layers.  gpu: bin/trace_run and
bin/generate as child processes on a small random checkpoint, against the plain oracle."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

from conftest import ROOT
from nanovllm_amd.engine.llm_engine import LLMEngine
from nanovllm_amd.model import registry
from nekodra_util import config, layer, moe, oracle_logits, random_checkpoint, rel_err
from oracle import ref_nekodra_modules

CFG = config([layer(heads=4, dim=16, vdim=8, rank=32, mlp=moe(experts=6, identity=2, top=3, ff=16, shared=24)), layer(heads=2, rank=20, mlp=None),
              layer(heads=3, rank=32, kv_from=0, mlp=moe(experts=3, identity=0, top=1, ff=12, shared=0))], vocab=61, width=40, positions=64)


def write_checkpoint(path, cfg, seed):
    ck = random_checkpoint(cfg, seed)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in ck.items()}, os.path.join(path, "model.safetensors"))
    return ck


def test_registry_builds_and_loads_a_checkpoint_directory(tmp_path):
    ck = write_checkpoint(str(tmp_path), CFG, seed=1)
    assert registry.architecture_of(registry.read_config(str(tmp_path))) == "Nekodra"
    model, cfg = registry.build_model(str(tmp_path), dtype=torch.float32, device="cpu", layers=ref_nekodra_modules)
    assert cfg.hidden_size == CFG["width"] and cfg.max_position_embeddings == 64
    l0, l1, l2 = model.layers
    assert l0.mlp.gate_up.shape == (6, 32, 40) and l0.mlp.router_weight.shape == (8, 40) and l0.mlp.shared_in.weight.shape == (48, 40)
    assert l0.mix.uk.weight.shape == (4, 32, 16) and l0.mix.uv.weight.shape == (4, 8, 32)
    torch.testing.assert_close(l0.mix.uk.weight[1], ck["l0.mix.uk"][16:32].float().t())
    assert l1.mlp is None and l1.norm2 is None and l2.mix.attn.latent_norm is None
    # one paged cache per layer with latents of its own; the sharing layer is bound to its source's
    assert [(s.key_dim, s.value_dim, s.value_in_key) for s in model.cache_specs()] == [(32, 32, True), (20, 20, True)]
    eng = LLMEngine(model, cfg, block_size=4, num_kvcache_blocks=16, device="cpu", max_num_seqs=2, dtype=torch.float32)
    assert model._caches[2][0].data_ptr() == model._caches[0][0].data_ptr() != model._caches[1][0].data_ptr()
    assert not eng.runner.has_state and eng.scheduler.prefix_caching
    toks = list(range(3, 30))
    got = eng.replay_step([("a", toks, list(range(len(toks))))], ["a"])
    assert rel_err(got, oracle_logits(CFG, ck, toks)) < 5e-5
    for gone in ("pos", "l0.norm1.b", "l0.norm2", "l0.mix.dkv", "l0.mix.dkv.norm", "l0.mix.sink", "l1.mix.g", "l2.mix.uk", "l0.mlp.e4.up",
                 "l0.mlp.router", "l0.mlp.shared.gate", "final.norm.b", "head"):
        with pytest.raises(KeyError):
            model.load_tensors({k: v for k, v in ck.items() if k != gone})
    with pytest.raises(KeyError):
        model.load_tensors({**ck, "l2.mix.dkv": torch.zeros(32, 40)})             # a sharing layer has no latent projection
    with pytest.raises(ValueError):
        model.load_tensors({**ck, "l0.mlp.e0.up": torch.zeros(17, 40)})
    with pytest.raises(ValueError):
        model.load_tensors({**ck, "l2.mix.uk": torch.zeros(30, 40)})
    # a checkpoint without a correction, and with one again
    model.load_tensors({k: v for k, v in ck.items() if not k.endswith("correction")})
    assert l0.mlp.router.correction is None
    model.load_tensors(ck)
    assert torch.equal(l0.mlp.router.correction, ck["l0.mlp.correction"].float())


def test_configurations_that_do_not_fit_the_design_are_refused():
    make = registry._REGISTRY["Nekodra"].make_config
    for layers in ([dict(layer(), type="no_such_mixer")], [layer(mlp={"kind": "no_such_kind"})], [layer(kv_from=0)], [layer(), layer(kv_from=1)],
                   [layer(rank=18), layer(rank=20, kv_from=0)], [layer(), layer(kv_from=0), layer(kv_from=1)],
                   [layer(mlp=moe(experts=2, identity=1, top=4))], [layer(mlp=moe(top=0))]):
        with pytest.raises(ValueError):
            make({**CFG, "layers": layers})
    bare = layer(mlp=moe(shared=0))
    del bare["mlp"]["router"]["identity"]
    assert make({**CFG, "layers": [bare]}).layers[0].mlp.identity == 0


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_replays_steps_and_writes_logits(tmp_path, dtype):
    model_dir, out_dir = str(tmp_path / "model"), str(tmp_path / "out")
    ck = write_checkpoint(model_dir, CFG, seed=2)
    a, b = list(range(5, 45)), [7, 7, 9, 11, 2, 60, 33]
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[17:19], "want": []}, {"id": "b", "tokens": b[:6], "want": [5]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[6:], "want": [0]}, {"id": "a", "tokens": a[19:], "want": [20, 0]}], "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [6]}], "end": ["c"]},      # reuses a's pages
    ]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", model_dir, "--dtype", dtype, "--out", out_dir,
                        "--max-tokens", "128", "--block-size", "16", "--max-seqs", "2"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    V = CFG["vocab"]
    la, lb = oracle_logits(CFG, ck, a), oracle_logits(CFG, ck, b)
    want = {0: [("a", 0), ("a", 16)], 1: [("b", 5)], 2: [("b", 6), ("a", 19 + 20), ("a", 19)], 3: [("b", 6)]}
    ref = {"a": la, "b": lb}
    bound = 5e-5 if dtype == "float32" else 3 * max(rel_err(oracle_logits(CFG, ck, a, torch.bfloat16), la),
                                                    rel_err(oracle_logits(CFG, ck, b, torch.bfloat16), lb))
    for n, rows in want.items():
        got = torch.from_numpy(np.fromfile(os.path.join(out_dir, f"{n}.f32"), dtype="<f4").reshape(-1, V).copy())
        assert got.shape[0] == len(rows)
        scale = la.pow(2).mean().sqrt()
        for g, (i, at) in zip(got, rows):
            d = g - ref[i][at]
            assert ((d - d.mean()).pow(2).mean().sqrt() / scale).item() < bound, (n, dtype)


@pytest.mark.gpu
def test_generate_program_matches_the_oracle_greedy(tmp_path):
    model_dir = str(tmp_path / "model")
    ck = write_checkpoint(model_dir, CFG, seed=3)
    prompt = [4, 8, 15, 16, 23, 42]
    p = subprocess.run([os.path.join(ROOT, "bin", "generate"), "--model", model_dir, "--dtype", "float32", "--prompt-ids",
                        ",".join(map(str, prompt)), "--max-tokens", "6", "--block-size", "16", "--max-seqs", "2", "--num-blocks", "8"],
                       capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    out = json.loads(p.stdout.splitlines()[0])
    seq = list(prompt)
    for _ in range(6):
        seq.append(int(oracle_logits(CFG, ck, seq)[-1].argmax()))
    assert out["token_ids"] == seq[len(prompt):]
