"""Vudivik on the HIP kernels (cuda:0): every mechanism alone and the engine scenarios of vudivik_cases.py against
the float64 oracle -- in fp32 (the kernels' 32-bit parts are then the whole computation: tight bounds) and in bf16
(the serving precision)."""
import numpy as np
import pytest
import torch

import test_vudivik as T
import vudivik_cases as C
import vudivik_oracle as O

pytestmark = pytest.mark.gpu

F32 = 5e-5   # fp32 GEMMs + fp32 kernels against float64
BF16 = 0.06  # bf16 GEMMs and activations
BOTH = [(torch.float32, F32), (torch.bfloat16, BF16)]


@pytest.fixture(autouse=True)
def _true_fp32():
    torch.backends.cuda.matmul.allow_tf32 = False
    yield


def _ties(dtype):
    """bf16 runs with a router leave out the few rows where rounding flips a nearly tied choice."""
    return C.near_ties(0.06 if dtype == torch.bfloat16 else 0.0)


def test_kernel_library_is_loaded():
    from githubrepostorag_amd.ops import _lib

    assert _lib.lib() is not None and _lib.loaded_path()
    for name in ("grag_causal_conv", "grag_chan_scan", "grag_moe_route", "grag_moe_align", "grag_moe_gemm", "grag_relu2",
                 "grag_postnorm_residual", "grag_rope_vnorm_store", "grag_sink_attn_prefill", "grag_sink_attn_decode"):
        assert hasattr(_lib.lib(), name)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 0.01)])
def test_boundary_alone(dtype, tol):
    T.boundary_case("cuda", dtype, tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_router_alone(dtype):
    T.router_case("cuda", dtype)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 0.02)])
def test_experts_alone(dtype, tol):
    # fp32: the plain tiles; bf16: the matrix-core tiles where the sizes are multiples of 8, small and (the last case,
    # 400 rows over 3 experts) large ones
    T.experts_case("cuda", dtype, tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_squared_relu_alone(dtype):
    T.relu2_case("cuda", dtype)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 5e-3)])
def test_rotary_alone(dtype, tol):
    T.rotary_case("cuda", dtype, tol)


@pytest.mark.parametrize("workgroups", [None, 1, 6, 12])
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 0.01)])
def test_scan_alone(dtype, tol, workgroups):
    T.scan_case("cuda", dtype, tol, workgroups)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 5e-3)])
def test_window_edges_in_prompts_and_decoding(dtype, tol):
    # (bf16: the stored output is rounded to 8 bits, 0.4 % of a marker up to 150; a wrong key is off by >= 1)
    C.case_window_edges("cuda", tol, dtype)
    C.case_window_edges("cuda", tol, dtype, bs=4, windows=(3, 4, 30))
    # several key tiles between the kept keys and the window; head sizes of the vector kernels
    C.case_window_edges("cuda", tol / 2, dtype, ctx=250, d=256, windows=(3, 64, 100), keeps=(0, 5, 64, 65, 130))
    C.case_window_edges("cuda", tol, dtype, ctx=150, d=152, windows=(3, 64), keeps=(5, 64, 65))


@pytest.mark.parametrize("mlp", [O.DENSE, O.MOE, None])
def test_single_layer_models(mlp):
    for dtype, tol in BOTH:
        with _ties(dtype):
            C.case_single_layer("cuda", tol, mlp, dtype)


@pytest.mark.parametrize("dtype,tol", BOTH)
@pytest.mark.parametrize("branch", ["left", "right"])
def test_one_branch_models(branch, dtype, tol):
    C.case_one_branch("cuda", tol, branch, dtype)


def test_shared_tensors():
    C.case_shared_tensors("cuda", F32)


@pytest.mark.parametrize("dtype,tol", BOTH)
def test_whole_prompt_and_layer_taps(dtype, tol):
    with _ties(dtype):
        C.case_whole_and_layers("cuda", tol if dtype == torch.float32 else 0.1, dtype)


@pytest.mark.parametrize("dtype,tol", BOTH)
def test_prefill_against_decode(dtype, tol):
    with _ties(dtype):
        C.case_prefill_vs_decode("cuda", tol, dtype)


@pytest.mark.parametrize("dtype,tol", BOTH)
def test_portions(dtype, tol):
    with _ties(dtype):
        C.case_portions("cuda", tol, dtype)


@pytest.mark.parametrize("dtype,tol", BOTH)
def test_unequal_batches(dtype, tol):
    if dtype == torch.bfloat16:
        with C.near_ties(0.06):
            C.case_batches("cuda", 0.03, dtype, alone=True)
    else:
        C.case_batches("cuda", tol, dtype)


def test_pages_and_slots_used_again():
    C.case_reuse("cuda", F32)


def test_other_sizes():
    C.case_other_sizes("cuda", F32)
    with C.near_ties(0.1):
        C.case_other_sizes("cuda", 0.15, torch.bfloat16)  # (tiny widths amplify the rounding)


def test_unlike_layers():
    C.case_mixed_layers("cuda", F32)


def test_first_tokens():
    C.case_first_tokens("cuda", F32)


def test_long_decode():
    C.case_long_decode("cuda", F32)


def test_sharp_softmax_picks_far_keys():
    C.case_sharp_far_keys("cuda", 5e-4)


def test_matrix_core_shapes_bf16():
    """Head sizes in multiples of 16, expert sizes in multiples of 8 and prompt portions of >= 16 queries: the bf16
    attention and expert kernels that run on the matrix cores, whole and in portions with decoded tokens at the end;
    a window of 70 and 24 kept positions against 64-key tiles."""
    cfg = O.make_config(width=64, mlps=(O.DENSE, O.MOE), heads=4, kv_heads=2, dim=32, vdim=48, scale=0.2, window=70, keep=24,
                        rot_dims=16, inner=128, state=16, dt_rank=8, experts=8, identity=1, top=3, expert_ff=40)
    sd = O.make_weights(cfg, seed=51)
    toks = C.tokens(cfg, 200, 8)
    want = O.forward(cfg, sd, toks)
    _, eng = C.build(cfg, sd, "cuda", torch.bfloat16)
    with C.near_ties(0.06):
        assert C.rel_err(C.feed_in_portions(eng, "w", toks, [200]), want) < BF16
        assert C.rel_err(C.feed_in_portions(eng, "c", toks, [64, 70, 50] + [1] * 16), want) < BF16


def test_serving_head_sizes():
    """The head sizes of the bench presets (128-wide attention heads, a state of 16, step sizes through more than 64
    numbers) at a small width, a window of 80, prompts and decoded tokens, both precisions."""
    cfg = O.make_config(width=128, vocab=128, mlps=(O.DENSE, None), heads=4, kv_heads=2, dim=128, vdim=128, scale=0.09,
                        window=80, keep=16, rot_dims=128, inner=256, state=16, dt_rank=96)
    sd = O.make_weights(cfg, seed=57)
    toks = C.tokens(cfg, 150, 11)
    want = O.forward(cfg, sd, toks)
    for dtype, tol in BOTH:
        _, eng = C.build(cfg, sd, "cuda", dtype)
        assert C.rel_err(C.feed_in_portions(eng, "c", toks, [70, 64] + [1] * 16), want) < tol


def test_key_splits_with_kept_tokens():
    """Decoding over the engine's key splits: the kept keys lie in the first split (or reach into the second), splits
    between them and the window are empty, the window starts inside a split.  A scale at which single keys stand out."""
    for window, keep in ((700, 20), (1100, 300), (1060, 16)):
        cfg = O.make_config(width=64, mlps=(None,), heads=4, kv_heads=2, dim=16, vdim=16, scale=2.0, window=window, keep=keep,
                            rot_dims=8, inner=64, state=16)
        sd = O.make_weights(cfg, seed=59)
        sd["l0.mix.right.out"] = torch.zeros_like(sd["l0.mix.right.out"])  # the attention alone
        toks = C.tokens(cfg, 1400, 12)
        want = O.forward(cfg, sd, toks)
        _, eng = C.build(cfg, sd, "cuda", torch.bfloat16, pool_tokens=1408)
        assert C.rel_err(C.feed_in_portions(eng, "k", toks, [1100] + [1] * 20 + [260] + [1] * 20), want) < BF16, (window, keep)


@pytest.mark.parametrize("graphs,mixed,window,max_batched", [(False, False, 1, 4096), (True, False, 1, 4096),
                                                             (True, False, 4, 4096), (False, True, 1, 8)])
def test_greedy_generation(graphs, mixed, window, max_batched):
    C.case_generate("cuda", graphs=graphs, mixed=mixed, window=window, max_batched=max_batched)


def test_bf16_batch_invariance():
    """bf16 serving: a request's logits beside other requests equal its logits alone (the same kernels see the
    same operands per row; only GEMM tiling may differ with the batch's row count)."""
    cfg = O.make_config(mlps=(O.DENSE, None))
    sd = O.make_weights(cfg, seed=37)
    a, b = C.tokens(cfg, 40, 1), C.tokens(cfg, 13, 2)
    _, eng = C.build(cfg, sd, "cuda", torch.bfloat16)
    alone = C.feed_in_portions(eng, "a", a, [40])
    o1 = eng.feed([("a2", a[:25], list(range(25))), ("b", b[:12], [])], [])
    o2 = eng.feed([("a2", a[25:], list(range(15))), ("b", b[12:], [0])], ["a2", "b"])
    assert C.rel_err(np.concatenate([o1, o2[:15]], 0), alone) < 0.02
