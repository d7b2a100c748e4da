"""Guzovik on the CPU (the engine's PyTorch op definitions, fp32) against the float64 oracle: mechanisms one by
one, then the engine's cache, batching and scheduler."""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import guzovik_cases as gc
import guzovik_oracle as go
from vllm_production_stack_amd.engine.config import EngineConfig, guzovik_config, guzovik_layers, resolve_model
from vllm_production_stack_amd.engine.llm_engine import LLMEngine
from vllm_production_stack_amd.models.latent_mixer import LatentAttention

DEV, DT, TOL = "cpu", "float32", 2e-5
CPU = torch.device("cpu")


# --------------------------------------------------------------------------- mechanisms
def test_residual_norms_and_layer_scale():
    gc.case_residual(CPU, DT, 2e-5)


def test_kv_write():
    gc.case_kv_write(CPU, DT)


def test_sliding_attention():
    gc.case_sliding_attention(CPU, DT, 2e-5, [(6, 2, 16, 24, 70), (3, 1, 5, 7, 33)])


def test_latent_window():
    gc.case_latent_window(CPU, DT, 2e-5, [(3, 40, 8, 45), (1, 9, 2, 3), (2, 24, 8, 1 << 30)])


def test_routing_mixture_and_clamped_unit():
    gc.case_routing(CPU)
    gc.case_mixture(CPU, DT, 2e-5, [(24, 12, 5, 2, 9, 16), (7, 5, 3, 1, 4, 0), (16, 8, 1, 1, 3, 3), (12, 10, 4, 4, 6, 5)])
    gc.case_clamped_unit(CPU, DT, 2e-5)


def test_rotation_of_neighbours_by_hand():
    """The oracle's rotation and visibility, written out for a small case."""
    x = torch.tensor([[1.0, 2.0, 3.0, 4.0, 5.0]], dtype=torch.float64)
    y = go.turn_neighbours(x, torch.tensor([3]), 100.0, 4)
    a, b = 3.0, 3.0 / 10.0
    want = [np.cos(a) - 2 * np.sin(a), 2 * np.cos(a) + np.sin(a), 3 * np.cos(b) - 4 * np.sin(b), 4 * np.cos(b) + 3 * np.sin(b), 5.0]
    assert torch.allclose(y[0], torch.tensor(want, dtype=torch.float64))
    assert go.visible(4, 2).int().tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
    p = go.weights_with_unit_sink(torch.zeros(1, 3, dtype=torch.float64), torch.tensor([[True, True, False]]))
    assert torch.allclose(p, torch.tensor([[1 / 3, 1 / 3, 0.0]], dtype=torch.float64))


def test_expanded_entries_cover_the_windows():
    """Pages a step expands: from the first key that its first row sees to its last row; every tile's pages are there."""
    model = LatentAttention()
    model.device = CPU
    pin = torch.Tensor.pin_memory
    torch.Tensor.pin_memory = lambda self: self
    try:
        for window in (0, 1, 63, 64, 65, 150, 10000):
            q_lens, ctx = [300, 2, 64], [1000, 130, 64]
            plan = model._plan_expanded(q_lens, ctx, 3, window)
            assert plan["total"] == 3 * sum(plan["n_pages"])
            for s, (n, c) in enumerate(zip(q_lens, ctx)):
                lo = max(0, c - n - window + 1) if window else 0
                assert plan["first"][s] == lo // 64 and plan["first"][s] + plan["n_pages"][s] == (c + 63) // 64
                for h in range(3):
                    run = plan["bt"][s * 3 + h, plan["first"][s]:(c + 63) // 64].tolist()
                    start = plan["base"][s] + h * plan["n_pages"][s]
                    assert run == list(range(start, start + plan["n_pages"][s]))
    finally:
        torch.Tensor.pin_memory = pin


# --------------------------------------------------------------------------- configuration and weights
def test_config_reader_and_loader(tmp_path):
    cfg = gc.config_a()
    w = go.make_weights(cfg)
    mc, _ = resolve_model(go.save_checkpoint(tmp_path / "m", cfg, w))
    assert mc.architecture == "guzovik" and mc.num_layers == 8 and mc.embedding_scale == 3.0 and mc.norm_eps == 1e-4
    s = mc.layer_specs
    assert [x.weights_of for x in s] == [None, None, 0, None, None, None, 1, 4] and s[3].mlp is None
    a, m = s[0].mixer, s[4].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.scale) == (6, 2, 16, 24, 70, 16 ** -0.5)
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.window, m.rope_base, m.scale) == (2, 8, 12, 16, 56, 130, 20000.0, 0.4)
    assert (s[0].mlp.experts, s[0].mlp.top, s[0].mlp.ff, s[0].mlp.shared_ff) == (7, 3, 24, 40) and s[4].mlp.shared_ff == 0
    assert (s[1].mlp.kind, s[1].mlp.ff, s[1].mlp.limit) == ("dense", 104, 0.8)
    stored = sum(v.numel() for k, v in w.items() if "norm" not in k and ".ls" not in k)
    assert mc.num_params() == stored and mc.prefill_flops()[0] > 0
    with pytest.raises(ValueError):
        guzovik_layers([{"type": "mingru", "mixer": {}, "mlp": None}])
    with pytest.raises(ValueError):
        guzovik_layers([go.attention(4, 2, 8, 8, 16, go.moe(8, 4, 5, 0))])
    with pytest.raises(ValueError):
        guzovik_layers([go.attention(4, 3, 8, 8, 16, None)])
    with pytest.raises(ValueError):
        guzovik_layers([go.latent(2, 8, 7, 8, 16, 10, None)])
    with pytest.raises(ValueError):
        guzovik_config("x", 10, 8, [go.attention(2, 1, 8, 8, 0, None)])
    one = go.attention(2, 1, 8, 8, 9, None)
    for bad in ([{**one, "weights_of": 0}], [{**one, "weights_of": 1}, {**one, "weights_of": 0}], [one, {**one, "weights_of": 2}],
                [one, {**go.attention(2, 1, 8, 8, 10, None), "weights_of": 0}]):
        with pytest.raises(ValueError):
            guzovik_layers(bad)
    chain = guzovik_layers([{**one, "weights_of": 2}, {**one, "weights_of": 0}, one])
    assert [x.weights_of for x in chain] == [2, 2, None]

    def refused(change):
        bad = dict(w)
        change(bad)
        folder = go.save_checkpoint(tmp_path / "bad", cfg, bad)
        with pytest.raises(ValueError):
            LLMEngine(EngineConfig(model=folder, dtype="float32", device="cpu", num_gpu_blocks_override=4, max_model_len=256))

    refused(lambda b: b.pop("l3.ls1"))
    refused(lambda b: b.pop("l0.mlp.shared.up"))
    refused(lambda b: b.__setitem__("l0.mix.g", b["l0.mix.g"][:-1]))
    refused(lambda b: b.__setitem__("l1.mix.uv", b["l1.mix.uv"][:-1]))
    refused(lambda b: b.__setitem__("l2.norm1", b["l0.norm1"]))      # layer 2 runs on layer 0's tensors
    refused(lambda b: b.__setitem__("l1.mix.sink", torch.zeros(3)))


def test_layers_that_share_tensors_have_entries_of_their_own(tmp_path):
    """One set of weights in memory, one part of the page per layer run."""
    cfg = gc.config_a()
    w = go.make_weights(cfg)
    eng = gc.make_engine(cfg, w, DEV, DT)
    model = eng.runner.model
    assert len(model.layers) == 5 and [li for li, _ in model.runs] == [0, 1, 0, 2, 3, 4, 1, 3]
    offs = [off for _, off in model.runs] + [model.page_elems]
    for (li, off), end in zip(model.runs, offs[1:]):
        m = model.layers[li].spec.mixer
        assert end - off == 64 * (m.kv_heads * (m.dim + m.vdim) if hasattr(m, "kv_heads") else m.kv_rank + m.rot_dim)
    eng.shutdown()


# --------------------------------------------------------------------------- the engine
@pytest.fixture(scope="module")
def model_a():
    cfg = gc.config_a()
    return cfg, go.make_weights(cfg, seed=3)


@pytest.fixture(scope="module")
def model_b():
    cfg = gc.config_b()
    return cfg, go.make_weights(cfg, seed=4)


def test_layers(model_a, model_b):
    gc.check_layers(DEV, DT, TOL, *model_a)
    gc.check_layers(DEV, DT, TOL, *model_b)


def test_whole_decode_and_portions(model_a):
    n = 150
    gc.check_cuts(DEV, DT, TOL, *model_a, n, [
        [n], [],                               # whole, token by token
        [n - 40],                              # a prompt, then decoded tokens
        [2, 2, 60, 1, 2, 61, 3, 2], [63, 2, 63, 2], [64, 64], [1, 127, 1, 1, 2]])


def test_other_sizes(model_b):
    gc.check_cuts(DEV, DT, TOL, *model_b, 131, [[131], [], [2, 62, 2, 63, 2], [65, 1, 1, 64]])


def test_first_tokens(model_a):
    for n in (1, 2, 3):
        gc.check_cuts(DEV, DT, TOL, *model_a, n, [[n], [], [1, n]], seed=n)


def test_long_decode(model_b):
    gc.check_cuts(DEV, DT, TOL, *model_b, 330, [[5]], pages=6)


def test_batches_and_reuse(model_a):
    gc.check_batches(DEV, DT, TOL, *model_a)


@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_window_edges(kind):
    for window in (1, 2, 64, 97):
        gc.check_window_edges(DEV, DT, TOL, kind, window)


def test_greedy_generation(model_a, model_b):
    gc.check_generate(DEV, DT, *model_a)
    gc.check_generate(DEV, DT, *model_b)
    gc.check_preemption(DEV, DT, *model_a)


def test_replay_command(tmp_path):
    """bin/trace_run: the line protocol, the logits files, requests that end and whose pages are used again."""
    cfg = gc.config_b()
    w = go.make_weights(cfg, seed=9)
    folder = go.save_checkpoint(tmp_path / "m", cfg, w)
    a, b = gc.tokens(cfg, 100, 1), gc.tokens(cfg, 70, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:64], "want": [0, 63]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[64:99], "want": []}, {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[3:], "want": [66]}, {"id": "a", "tokens": a[99:], "want": [0]}], "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "c", "tokens": a, "want": [99]}], "end": ["c"]},  # its pages were a's or b's
    ]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "256", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    la, lb = go.forward(cfg, w, a), go.forward(cfg, w, b)
    want = {0: la[[0, 63]], 1: lb[[2]], 2: torch.stack([lb[69], la[99]]), 3: la[[99]]}
    for n, ref in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
        assert got.shape == ref.shape and go.row_errors(got, ref).max().item() < TOL
