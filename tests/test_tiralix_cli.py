"""Tiralix from a checkpoint directory: config.json -> registry -> model, *.safetensors -> parameters, and the two
command-line programs.  CPU: the registry and loader with the eager stand-in layers.  gpu: bin/trace_run and
bin/generate as child processes on a small random checkpoint, against the plain oracle."""
import copy
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
from oracle import ref_tiralix_modules
from tiralix_util import config, dense, mamba_layer, oracle_logits, parallel_layer, random_checkpoint, rel_err

CFG = config([parallel_layer(heads=4, kv_heads=2, dim=16, vdim=24, rot_dims=8, rheads=3, rdim=16, rvdim=8), mamba_layer(mlp=None),
              mamba_layer(inner=32, state=8, dt_rank=4, conv=4, mlp=dense(48))], vocab=61, width=40)


def write_checkpoint(path, cfg, seed):
    ck = random_checkpoint(cfg, seed)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in ck.items()}, os.path.join(path, "model.safetensors"))
    return ck


def test_registry_builds_and_loads_a_checkpoint_directory(tmp_path):
    ck = write_checkpoint(str(tmp_path), CFG, seed=1)
    assert registry.architecture_of(registry.read_config(str(tmp_path))) == "Tiralix"
    model, cfg = registry.build_model(str(tmp_path), dtype=torch.float32, device="cpu", layers=ref_tiralix_modules)
    assert cfg.hidden_size == CFG["width"] and cfg.logit_scale == CFG["logit_scale"] and cfg.logit_softcap == CFG["logit_softcap"]
    mix = model.layers[0].mix
    assert mix.o.weight.shape == (40, 4 * 24 + 3 * 8) and mix._fused_w.shape[0] % 8 == 0
    torch.testing.assert_close(mix.o.weight[:, 96:], ck["l0.mix.right.o"].float())
    torch.testing.assert_close(model.layers[0].norm2.applied, ck["l0.norm2"].float() * ck["l0.ls2"].float())
    torch.testing.assert_close(mix._fused_w[:64], ck["l0.mix.left.q"].float())
    assert model.layers[1].norm2 is None and model.layers[1].mlp is None
    kinds = [type(s).__name__ for s in model.cache_specs()]
    assert kinds == ["PagedKVSpec", "SlotStateSpec", "SlotStateSpec", "SlotStateSpec"]
    toks = list(range(3, 30))
    for _ in range(2):                                        # a loaded model can be loaded again (the inputs are fused by then)
        eng = LLMEngine(model, cfg, block_size=4, num_kvcache_blocks=16, device="cpu", max_num_seqs=2, dtype=torch.float32)
        got = eng.replay_step([("a", toks, list(range(len(toks))))], ["a"])
        assert rel_err(got, oracle_logits(CFG, ck, toks)) < 5e-5
        ck = random_checkpoint(CFG, seed=7)
        model.load_tensors(ck)
    for gone in ("l0.mix.left.q.norm", "l0.mix.left.o", "l0.mix.right.o", "l0.mix.right.norm", "l0.ls1", "l0.mlp.up", "l1.mix.A_log",
                 "l1.mix.conv.b", "l2.mix.dt.b", "final.norm"):
        with pytest.raises(KeyError):
            model.load_tensors({k: v for k, v in ck.items() if k != gone})
    with pytest.raises(KeyError):
        model.load_tensors({**ck, "l1.norm2": torch.zeros(40)})             # a layer without feed-forward has no second norm
    for name in ("l0.mix.left.o", "l0.mlp.gate", "l2.mix.x"):
        with pytest.raises(ValueError):
            model.load_tensors({**ck, name: torch.zeros(17, 40)})
    make = registry._REGISTRY["Tiralix"].make_config

    def broken(change):
        c = copy.deepcopy(CFG)
        change(c["layers"])
        return c
    for change in (lambda L: L[0].update(type="no_such_mixer"), lambda L: L[0]["mlp"].update(kind="no_such_kind"),
                   lambda L: L[0]["mixer"]["left"].update(heads=3), lambda L: L[0]["mixer"]["left"]["rot"].update(dims=18),
                   lambda L: L[0]["mixer"]["left"]["rot"].update(dims=7), lambda L: L[0]["mixer"]["right"].update(decay=[0.5]),
                   lambda L: L[1]["mixer"].update(conv=0)):
        with pytest.raises(ValueError):
            make(broken(change))


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
        {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [6]}], "end": ["c"]},      # reuses a's pages and slot
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


def test_launch_plans_of_any_size_are_answered():
    """The workspace queries plan a launch on the host: few channels, long portions, many sequences and one."""
    from nanovllm_amd import _lib
    dll = _lib.mixers()
    for B, rest, lead in ((1, 0, 0), (2, 1, 1), (70, 69, 0), (300, 2000, 250)):
        for mq in (1, 2, 16, 17, 255, 256, 512, 1000, 100000):
            T = mq + rest
            for C, N in ((1, 1), (7, 3), (24, 6), (100, 256), (20000, 16)):
                assert 0 <= dll.nv_selective_scan_workspace_bytes(B, T, C, N, mq, lead) <= 4 * (2 * 16 * T // mq + 2) * C * (N + 1)
            for H, Dk, Dv in ((1, 1, 1), (3, 5, 65), (64, 128, 256)):
                assert 0 <= dll.nv_fixed_decay_workspace_bytes(B, T, H, Dk, Dv, mq, lead, 0) <= 4 * (2 * 16 * T // mq + 2) * H * Dk * Dv
                assert dll.nv_fixed_decay_workspace_bytes(B, T, H, Dk, Dv, mq, lead, 1) == 0        # float32 rows run token by token
    assert dll.nv_selective_scan_workspace_bytes(5, 5, 64, 16, 1, 5) == dll.nv_fixed_decay_workspace_bytes(5, 5, 2, 32, 32, 1, 5, 0) == 0
