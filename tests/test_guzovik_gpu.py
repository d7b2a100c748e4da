"""Guzovik on the GPU: the HIP kernels one by one against float64 definitions in both activation dtypes,
then the engine in fp32 and in bf16 against the float64 oracle (same cases as on the CPU), and HIP-graph
decode steps against eager ones."""

import functools

import pytest
import torch

import guzovik_cases as gc
import guzovik_oracle as go
from vllm_production_stack_amd import ops
from vllm_production_stack_amd.engine.request import SamplingParams

pytestmark = pytest.mark.gpu

# 16-bit runs choose every unit (``steady``): a routing decision that rounding turns over changes its row and every row
# that attends to it, and says nothing about the kernels; fp32 is the sharp run
MODES = [("float32", 5e-5, 0), ("bfloat16", 0.12, 3)]
BOTH = ["float32", "bfloat16"]
KERNEL_TOL = {"float32": 2e-5, "bfloat16": 2e-2}
DEV = torch.device("cuda")


@functools.lru_cache(maxsize=None)
def model(name, dtype="float32"):
    cfg = {"a": gc.config_a, "b": gc.config_b, "c": gc.config_c}[name]()
    if dtype == "bfloat16":
        cfg = gc.steady(cfg)
    return cfg, go.make_weights(cfg, seed={"a": 3, "b": 4, "c": 5}[name])


@pytest.mark.parametrize("dtype", BOTH)
def test_residual_norms_and_layer_scale(dtype):
    gc.case_residual(DEV, dtype, KERNEL_TOL[dtype])
    assert ops.native_loaded()


@pytest.mark.parametrize("dtype", BOTH)
def test_kv_write(dtype):
    gc.case_kv_write(DEV, dtype)


@pytest.mark.parametrize("dtype", BOTH)
def test_sliding_attention(dtype):
    gc.case_sliding_attention(DEV, dtype, KERNEL_TOL[dtype], [(6, 2, 16, 24, 70), (3, 1, 5, 7, 33), (2, 2, 200, 130, 129)])


@pytest.mark.parametrize("shape", [(4, 2, 64, 64, 70), (6, 2, 64, 96, 128), (5, 1, 96, 96, 63), (6, 3, 96, 192, 64),
                                   (8, 1, 128, 128, 500), (2, 2, 128, 320, 65)])
def test_sliding_attention_on_the_matrix_cores(shape):
    """Key widths 64, 96 and 128, value widths in one chunk of channels and in several."""
    heads, kv, dim, vdim, _ = shape
    assert ops.window_mfma_supported(heads, kv, dim, vdim, True)
    gc.case_sliding_attention(DEV, "bfloat16", 2e-2, [shape])


@pytest.mark.parametrize("dtype", BOTH)
def test_latent_window(dtype):
    gc.case_latent_window(DEV, dtype, KERNEL_TOL[dtype], [(3, 40, 8, 45), (1, 9, 2, 3), (2, 300, 10, 257), (2, 24, 8, 1 << 30)])


@pytest.mark.parametrize("shape", [(3, 64, 32, 150), (16, 128, 64, 64), (5, 512, 64, 65), (70, 64, 64, 100), (2, 128, 192, 1),
                                   (4, 64, 96, 1 << 30)])
def test_latent_window_on_the_matrix_cores(shape):
    assert ops.latent_mfma_supported(*shape[1:3])
    gc.case_latent_window(DEV, "bfloat16", 2e-2, [shape])


def test_expanded_entries():
    shapes = [(32, 64, 50), (64, 96, 65), (64, 128, 1), (128, 128, 64), (128, 192, 1 << 30)]
    assert all(ops.latent_expanded_supported(v, k) for v, k, _ in shapes)
    gc.case_expanded_entries(DEV, shapes)


@pytest.mark.parametrize("dtype", BOTH)
def test_routing_mixture_and_clamped_unit(dtype):
    gc.case_routing(DEV)
    tol = 3e-5 if dtype == "float32" else 4e-2
    gc.case_mixture(DEV, dtype, tol, [(24, 12, 5, 2, 9, 16), (7, 5, 3, 1, 4, 0), (64, 96, 4, 2, 70, 64), (64, 128, 4, 4, 9, 32)])
    gc.case_clamped_unit(DEV, dtype, tol)


@pytest.mark.parametrize("tokens", [1, 5, 20, 40, 100])
def test_mixture_on_the_matrix_cores(tokens):
    """The weight-streaming kernels of decode-sized batches (also for more experts than a top-k kernel keeps in
    registers) and the grouped prefill GEMM."""
    assert ops.moe_mfma_supported(128, 512)
    gc.case_mixture(DEV, "bfloat16", 4e-2, [(128, 512, 6, 2, tokens, 256), (128, 64, 3, 3, tokens, 0), (128, 512, 80, 3, tokens, 0)])


@pytest.mark.parametrize("dtype,tol,loose", MODES)
def test_layers(dtype, tol, loose):
    gc.check_layers("cuda", dtype, tol, *model("a", dtype))
    gc.check_layers("cuda", dtype, tol, *model("b", dtype))
    gc.check_layers("cuda", dtype, tol, *model("c", dtype))


@pytest.mark.parametrize("dtype,tol,loose", MODES)
def test_whole_decode_and_portions(dtype, tol, loose):
    gc.check_cuts("cuda", dtype, tol, *model("a", dtype), 150, [[150], [], [118], [64, 64], [63, 2, 63, 2], [2, 2, 60, 1, 2, 61, 3, 2],
                                                      [1, 1, 1, 25, 23, 2]], loose=loose)


@pytest.mark.parametrize("dtype,tol,loose", MODES)
def test_other_sizes_and_first_tokens(dtype, tol, loose):
    tol = tol if dtype == "float32" else 0.15   # a width of 45 averages bf16 rounding over few terms
    gc.check_cuts("cuda", dtype, tol, *model("b", dtype), 160, [[160], [1], [2, 1, 2], [5, 2, 7, 1, 70, 2, 64], [128, 2]], loose=loose)
    for n in (1, 2, 3):
        gc.check_cuts("cuda", dtype, tol, *model("b", dtype), n, [[n], [], [1, n]], seed=n, loose=loose)


@pytest.mark.parametrize("dtype,tol,loose", MODES)
def test_tiled_kernels_in_the_engine(dtype, tol, loose):
    """The attention tile kernels, in latent space and, for parts of 256 rows and more, over expanded heads (from the
    middle of a context: pages before the window are not expanded); grouped and weight-streaming units."""
    cfg, w = model("c", dtype)
    assert ops.latent_mfma_supported(64, 32) and ops.latent_mfma_supported(128, 64) and ops.latent_mfma_supported(64, 96)
    gc.check_cuts("cuda", dtype, tol, cfg, w, 640, [[640], [300, 340], [130, 1, 1, 268], [620], [330, 290]], loose=loose)


@pytest.mark.parametrize("dtype,tol,loose", MODES)
def test_long_decode(dtype, tol, loose):
    gc.check_cuts("cuda", dtype, tol, *model("a", dtype), 330, [[20]], pages=6, loose=loose)
    gc.check_cuts("cuda", dtype, tol, *model("c", dtype), 330, [[20]], pages=6, loose=loose)


@pytest.mark.parametrize("dtype,tol,loose", MODES)
def test_batches_and_reuse(dtype, tol, loose):
    gc.check_batches("cuda", dtype, tol, *model("a", dtype), loose=loose)
    gc.check_batches("cuda", dtype, tol, *model("c", dtype), loose=loose)


@pytest.mark.parametrize("kind", ["attention", "latent"])
@pytest.mark.parametrize("dtype,tol", [("float32", 5e-5), ("bfloat16", 0.15)])
def test_window_edges(dtype, tol, kind):
    for window in (1, 64, 97):
        gc.check_window_edges("cuda", dtype, tol, kind, window)


def test_greedy_generation():
    gc.check_generate("cuda", "float32", *model("a"))
    gc.check_generate("cuda", "float32", *model("b"))
    gc.check_preemption("cuda", "float32", *model("a"))


@pytest.mark.parametrize("dtype", BOTH)
def test_decode_graphs_match_eager(dtype):
    """Decode steps replayed from HIP graphs (positions and pages are graph inputs) give the tokens of eager steps,
    replay after replay, with eager prefill steps of new requests in between."""
    cfg, w = model("c", dtype)
    prompts = [gc.tokens(cfg, n, 90 + n) for n in (170, 3, 33, 64, 20, 9)]
    params = SamplingParams(max_tokens=40, temperature=0.0, ignore_eos=True)
    outs = {}
    for eager in (True, False):
        eng = gc.make_engine(cfg, w, "cuda", dtype, pages=16, slots=3, budget=64, eager=eager)
        outs[eager] = eng.generate(prompts, params)
        if not eager and dtype == "bfloat16":
            assert eng.runner.model.graph_capturable and eng.runner.step_kinds["decode_graph"] > 20
        eng.shutdown()
    assert outs[True] == outs[False]
    if dtype == "float32":
        assert outs[True][0] == go.greedy(cfg, w, prompts[0], 40)


def test_preset_at_random_weights_generates():
    from vllm_production_stack_amd.engine.config import EngineConfig
    from vllm_production_stack_amd.engine.llm_engine import LLMEngine

    eng = LLMEngine(EngineConfig(model="tiny-guzovik", dtype="bfloat16", max_model_len=512, max_num_seqs=4,
                                 num_gpu_blocks_override=16, enable_prefix_caching=False))
    prompts = [[5, 6, 7] * 100, [9] * 3]
    greedy = SamplingParams(max_tokens=8, temperature=0.0, ignore_eos=True)
    outs = eng.generate(prompts, greedy)
    assert [len(o) for o in outs] == [8, 8]
    drawn = eng.generate(prompts, SamplingParams(max_tokens=8, temperature=0.9, top_p=0.9, seed=5, ignore_eos=True))
    assert [len(o) for o in drawn] == [8, 8]
    assert eng.sleep(1) > 0
    eng.wake_up()
    assert eng.generate(prompts, greedy) == outs
    eng.shutdown()
