"""Kapanex on the HIP kernels (cuda:0): every mechanism alone and the engine scenarios of kapanex_cases.py against
the float64 oracle -- in fp32 (the kernels' 32-bit parts are then the whole computation: tight bounds) and in bf16
(the serving precision)."""
import numpy as np
import pytest
import torch

import kapanex_cases as C
import kapanex_oracle as O
import test_kapanex as T

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
    for name in ("grag_causal_conv", "grag_delta_scan", "grag_delta_step", "grag_gated_rmsnorm", "grag_moe_route",
                 "grag_moe_align", "grag_moe_gemm", "grag_residual_layernorm", "grag_rope_vnorm_store",
                 "grag_sink_attn_prefill", "grag_sink_attn_decode"):
        assert hasattr(_lib.lib(), name)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 0.005)])
def test_boundary_alone(dtype, tol):
    T.boundary_case("cuda", dtype, tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_router_alone(dtype):
    T.router_case("cuda", dtype)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 5e-3)])
def test_rotary_alone(dtype, tol):
    T.rotary_case("cuda", dtype, tol)


@pytest.mark.parametrize("size", range(len(T.DELTA_SIZES)))
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 5e-5), (torch.bfloat16, 0.01)])
def test_delta_rule_alone(size, dtype, tol):
    """bf16: q, k, v are the bf16 output of the convolution (whose rounding may fall to either side of a tie), everything
    after it is fp32."""
    T.delta_case("cuda", dtype, tol, T.DELTA_SIZES[size:size + 1])


def test_delta_rule_crafted():
    """A single write at the start that the last token asks for, the same key many times over, decays of 1."""
    for dtype, tol in ((torch.float32, 2e-3), (torch.bfloat16, 0.02)):
        T.delta_case("cuda", dtype, tol, T.DELTA_SIZES[:2] + T.DELTA_SIZES[5:6], crafted=True)


def test_delta_rule_is_fp32_in_bf16_runs():
    """On the same bf16 inputs the bf16 kernels (exact bf16 products, fp32 operands in three parts) and the fp32 kernels
    agree to fp32 rounding, in the state as well."""
    from githubrepostorag_amd.ops.recurrent import gated_delta
    from test_pubulix import _meta

    for H, G, d, vd in ((4, 2, 128, 128), (3, 1, 40, 24), (2, 2, 200, 72)):
        g = torch.Generator().manual_seed(d)
        n, vv = 300, H * vd
        xc = torch.randn(n, 2 * G * d + vv, generator=g).to(torch.bfloat16).cuda()
        p = torch.randn(n, vv + 2 * H, generator=g).to(torch.bfloat16).cuda()
        alog, dtb, w = torch.full((H,), -3.0).cuda(), torch.zeros(H).cuda(), torch.ones(vv).cuda()
        out = []
        for dt in (torch.bfloat16, torch.float32):
            st = torch.zeros(2, H, d, vd, device="cuda")
            gated_delta(xc.to(dt), p.to(dt), vv, vv + H, 0, alog, dtb, w, 1e-6, st, _meta("cuda", [n], [n], [1]), H, G, d, vd)
            out.append(st[1].double())
        assert float((out[0] - out[1]).abs().max() / out[1].abs().max()) < 3e-6, (H, d)


@pytest.mark.parametrize("alog", [-6.0, 1.0, 5.0])
def test_delta_rule_over_many_chunks(alog):
    """Portions of ten chunks and of one and a half beside each other, behind a state that an earlier portion left: decays
    that keep everything, that forget within a chunk, and that underflow to 0 within a token or two."""
    from githubrepostorag_amd.ops.recurrent import gated_delta
    from test_pubulix import _meta

    H, G, d, vd, lens = 3, 1, 48, 40, ((7, 70), (640, 97), (33, 129))
    vv = H * vd
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-5)):
        g = torch.Generator().manual_seed(5)
        ab, dtb, w = torch.full((H,), alog), torch.randn(H, generator=g), torch.ones(vv)
        st = torch.randn(3, H, d, vd, generator=g).cuda()
        hist, cur = [[], []], [0, 0]
        for ls in lens:
            xs = [torch.randn(n, 2 * G * d + vv, generator=g).to(dtype) for n in ls]
            ps = [torch.randn(n, vv + 2 * H, generator=g).to(dtype) for n in ls]
            for s in (0, 1):
                hist[s].append((xs[s], ps[s]))
                cur[s] += ls[s]
            gated_delta(torch.cat(xs).cuda(), torch.cat(ps).cuda(), vv, vv + H, 0, ab.cuda(), dtb.cuda(), w.cuda(), 1e-6, st,
                        _meta("cuda", ls, cur, [2, 1]), H, G, d, vd)
        for s in (0, 1):
            x, p = (torch.cat([h[i] for h in hist[s]]).double() for i in (0, 1))
            q, k = (O.unit(x[:, i * G * d:(i + 1) * G * d].view(-1, G, d)).repeat_interleave(H // G, dim=1) for i in (0, 1))
            dec = torch.exp(-torch.exp(ab.double()) * O.softplus(p[:, vv + H:] + dtb.double()))
            _, S = O.delta_rule(q, k, x[:, 2 * G * d:].view(-1, H, vd), dec, torch.sigmoid(p[:, vv:vv + H]))
            err = float((st[2 - s].cpu().double() - S).abs().max() / S.abs().max())
            assert err < tol, (dtype, s, err)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 5e-3)])
def test_window_edges_in_prompts_and_decoding(dtype, tol):
    # (bf16: the stored output is rounded to 8 bits, 0.4 % of a marker up to 150; a wrong key is off by >= 1)
    C.case_window_edges("cuda", tol, dtype)
    C.case_window_edges("cuda", tol, dtype, bs=4, windows=(3, 4, 30))
    C.case_window_edges("cuda", tol / 2, dtype, ctx=250, d=256, windows=(3, 64, 100))


@pytest.mark.parametrize("kind", [O.DELTA, O.ATT])
@pytest.mark.parametrize("moe", [True, False])
def test_single_layer_models(kind, moe):
    for dtype, tol in BOTH:
        with _ties(dtype):
            C.case_single_layer("cuda", tol, kind, moe, dtype)


@pytest.mark.parametrize("dtype,tol", BOTH)
def test_whole_prompt_and_layer_taps(dtype, tol):
    with _ties(dtype):
        C.case_whole_and_layers("cuda", tol if dtype == torch.float32 else 0.1, dtype)


def test_shared_tensors():
    C.case_shared_tensors("cuda", F32)


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
        C.case_batches("cuda", tol, dtype, long=5)  # several chunks of several sequences in one step


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
    attention and expert kernels that run on the matrix cores, whole and in portions with decoded tokens at the end; a
    window of 70 against 64-key tiles."""
    cfg = O.make_config(width=64, mixers=(O.DELTA, O.ATT), heads=4, kv_heads=2, dim=32, vdim=48, scale=0.7, window=70,
                        rot_dims=16, dheads=4, dkv_heads=2, ddim=32, dvdim=48, experts=8, groups=(4, 2), top=3, ff=40,
                        shared_ff=24)
    sd = O.make_weights(cfg, seed=51)
    toks = C.tokens(cfg, 200, 8)
    want = O.forward(cfg, sd, toks)
    _, eng = C.build(cfg, sd, "cuda", torch.bfloat16)
    with C.near_ties(0.06):
        assert C.rel_err(C.feed_in_portions(eng, "w", toks, [200]), want) < BF16
        assert C.rel_err(C.feed_in_portions(eng, "c", toks, [64, 70, 50] + [1] * 16), want) < BF16


def test_serving_head_sizes():
    """The head sizes of the bench presets (128-wide heads in both mixers) at a small width, a window of 80, prompts and
    decoded tokens, both precisions."""
    cfg = O.make_config(width=128, vocab=128, mixers=(O.DELTA, O.ATT, O.DELTA), moe=False, heads=4, kv_heads=2, dim=128,
                        vdim=128, scale=0.2, window=80, rot_dims=128, dheads=4, dkv_heads=2, ddim=128, dvdim=128, conv=4)
    sd = O.make_weights(cfg, seed=57)
    toks = C.tokens(cfg, 150, 11)
    want = O.forward(cfg, sd, toks)
    for dtype, tol in BOTH:
        _, eng = C.build(cfg, sd, "cuda", dtype)
        assert C.rel_err(C.feed_in_portions(eng, "c", toks, [70, 64] + [1] * 16), want) < tol


@pytest.mark.parametrize("graphs,mixed,window,max_batched", [(False, False, 1, 4096), (True, False, 1, 4096),
                                                             (True, False, 4, 4096), (False, True, 1, 8)])
def test_greedy_generation(graphs, mixed, window, max_batched):
    C.case_generate("cuda", graphs=graphs, mixed=mixed, window=window, max_batched=max_batched)


def test_bf16_batch_invariance():
    """bf16 serving: a request's logits beside other requests equal its logits alone (the same kernels see the
    same operands per row; only GEMM tiling may differ with the batch's row count)."""
    cfg = O.make_config(moe=False)
    sd = O.make_weights(cfg, seed=37)
    a, b = C.tokens(cfg, 40, 1), C.tokens(cfg, 13, 2)
    _, eng = C.build(cfg, sd, "cuda", torch.bfloat16)
    alone = C.feed_in_portions(eng, "a", a, [40])
    o1 = eng.feed([("a2", a[:25], list(range(25))), ("b", b[:12], [])], [])
    o2 = eng.feed([("a2", a[25:], list(range(15))), ("b", b[12:], [0])], ["a2", "b"])
    assert C.rel_err(np.concatenate([o1, o2[:15]], 0), alone) < 0.02
