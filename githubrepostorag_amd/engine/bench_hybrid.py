"""``bench.py --hybrid [zofesun|namudra|leripel|pubulix|vudivik|kapanex]``: prefill and decode throughput of a hybrid decoder beside the decoders of
equal size that the engine already serves (same width, heads, head size, FFN width, layer count, vocabulary; random
weights, synthetic token ids), all through LLMEngine.generate, and a per-kernel table: each new kernel and the
like kernel of the closest model as a fraction of the roofline of what bounds it (HBM bytes or matrix / vector
flops).  Zofesun stands beside Qwen2; Namudra beside Zofesun (the closest: fp32 residual, decay scan, sink
attention kernels) and Qwen2; Leripel beside Namudra (the closest: fp32 residual, retention scan, the same attention
kernel family, a layer list that is data) and Qwen2; Pubulix beside Leripel (the closest: the same attention kernels
with a window instead of blocks, experts on the same grouped GEMM, the same convolution and boundary kernels) and
Qwen2, with Namudra's latent attention as the like kernel of its latent layers; Vudivik beside Leripel (the closest: a
state-space scan behind the same convolution, routed experts on the same grouped GEMM, the same attention kernels) and
Qwen2, with Pubulix's window attention as the like kernel of its own; Kapanex beside Leripel (the closest: one scan, one
attention layer in turn, side-by-side sublayers, grouped experts with a gated shared one) and Qwen2, with Pubulix's window
attention and Vudivik's normed rotary store as the like kernels of its own."""
from __future__ import annotations

import json
import time

import torch

HBM_BPS = 8.0e12        # HBM3E
MFMA_BF16 = 2.5e15      # dense bf16 matrix flop/s
VALU_F32 = 1.57e14      # fp32 vector flop/s (fma = 2)

SIZES = {
    # name: (width, heads, kv_heads, head size, ffn, layers, mingru every)
    "1b-like": (1536, 12, 2, 128, 8960, 8, 4),
    "7b-like": (3584, 28, 4, 128, 18944, 4, 4),
}
VOCAB = 32768


def _timed(fn, iters=10, warm=2):
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    e0.record()
    for _ in range(iters):
        fn()
    e1.record()
    torch.cuda.synchronize()
    return e0.elapsed_time(e1) * 1e-3 / iters


def _models(name, dev):
    from ..models.configs import DecoderConfig, zofesun_config
    from ..models.qwen2 import Qwen2Model
    from ..models.zofesun import ZofesunModel

    W, H, G, D, ff, nl, every = SIZES[name]
    zc = zofesun_config(f"zofesun-{name}", VOCAB, W, nl, heads=H, kv_heads=G, dim=D, vdim=D, lin_heads=H, lin_dim=D,
                        lin_vdim=D, ff=ff, mingru_every=every)
    qc = DecoderConfig(f"qwen2-{name}", VOCAB, W, ff, nl, H, G, D, max_position=32768)
    return (lambda: ZofesunModel(zc, device=dev, seed=1)), (lambda: Qwen2Model(qc, device=dev, seed=1))


def _namudra_models(name, dev):
    """Namudra at a bench size: per four layers retention, windowed sigmoid attention, latent attention, windowed
    attention (every layer with a feed-forward, two residual streams), beside the Zofesun and Qwen2 stacks."""
    from ..models.configs import namudra_config
    from ..models.namudra import NamudraModel

    W, H, G, D, ff, nl, _ = SIZES[name]
    nc = namudra_config(f"namudra-{name}", VOCAB, W, ("rala" * nl)[:nl], heads=H, kv_heads=G, dim=D, ff=ff,
                        window=1024, kv_rank=192, q_rank=W // 4, rot_dim=64, streams=2, ret_ff=True)
    mk_z, mk_q = _models(name, dev)
    return (lambda: NamudraModel(nc, device=dev, seed=1)), mk_z, mk_q


def _engine_numbers(make, dev, batch, prompt_len, gen_len, graphs=True):
    from .llm_engine import EngineConfig, LLMEngine
    from .sequence import SamplingParams

    model = make()
    need = batch * (prompt_len + gen_len + 16)
    eng = LLMEngine(model, None, EngineConfig(max_num_seqs=batch, max_model_len=prompt_len + gen_len + 16,
                                              max_num_batched_tokens=max(8192, prompt_len), num_blocks=need // 16 + 2,
                                              use_cuda_graph=graphs, enable_prefix_caching=False))
    g = torch.Generator().manual_seed(0)
    prompts = [torch.randint(0, VOCAB, (prompt_len,), generator=g).tolist() for _ in range(batch)]

    def run(n):
        t0 = time.perf_counter()
        eng.generate(prompts, SamplingParams(max_tokens=n, temperature=0.0, ignore_eos=True))
        torch.cuda.synchronize()
        return time.perf_counter() - t0

    run(2)  # compile / capture
    run(gen_len + 1)
    t_pre = min(run(1) for _ in range(2))
    t_all = min(run(gen_len + 1) for _ in range(2))
    out = {"prefill_tok_s": round(batch * prompt_len / t_pre), "decode_tok_s": round(batch * gen_len / max(t_all - t_pre, 1e-9)),
           "prefill_ms": round(t_pre * 1e3, 2), "decode_ms_per_step": round((t_all - t_pre) / gen_len * 1e3, 3)}
    del eng, model
    torch.cuda.empty_cache()
    return out


def _kernel_table(dev, H=28, G=4, D=128, W=3584, ff=18944, T=2048, B=64, ctx=2048, bs=16):
    """[(kernel, seconds, bound, fraction of roofline)] for the new kernels and the like kernels of Qwen2."""
    from ..ops.attention import AttnMetadata, paged_attention, sink_attention
    from ..ops.elementwise import (clamped_glu, qkv_rope_kvstore, rope_cos_sin, rope_table, rope_vnorm_store, silu_mul)
    from ..ops.norm import dyt_residual, rmsnorm
    from ..ops.recurrent import decay_attention, gated_rmsnorm, mingru_scan

    bf = torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    rows = []

    def add(name, sec, flops=0.0, bytes_=0.0, peak=MFMA_BF16):
        t_c, t_m = flops / peak, bytes_ / HBM_BPS
        bound = "flops" if t_c >= t_m else "bytes"
        rows.append({"kernel": name, "us": round(sec * 1e6, 1), "bound": bound,
                     "roofline_fraction": round(max(t_c, t_m) / sec, 4)})

    # ---- prefill attention: one prompt of T tokens
    nb = T // bs
    kc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    vc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    q = torch.randn(T, H, D, device=dev).to(bf)
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([0], **i32))
    sinks = torch.zeros(H, device=dev)
    fl = 4.0 * T * T / 2 * H * D
    add("sink_attn_prefill", _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, sinks)), flops=fl)
    add("qwen2 paged_attention prefill", _timed(lambda: paged_attention(q, kc, vc, meta, 0.09)), flops=fl)
    # ---- decode attention: B rows of ctx keys
    nbd = ctx // bs
    kd = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    vd_ = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    qd = torch.randn(B, H, D, device=dev).to(bf)
    part_o = torch.empty(8 * B * H * D, device=dev)
    part_ml = torch.empty(8 * B * H * 2, device=dev)
    dmeta = AttnMetadata(q_start=torch.arange(B + 1, **i32), ctx_len=torch.full((B,), ctx, **i32),
                         block_tables=(torch.arange(B * nbd, **i32) + 1).view(B, nbd), slot_mapping=None, max_q_len=1,
                         num_seqs=B, num_tokens=B, is_decode=True, num_splits=8, split_len=ctx // 8, part_o=part_o,
                         part_ml=part_ml, state_slots=torch.arange(B, **i32))
    by = 2.0 * B * ctx * G * D * 2
    add("sink_attn_decode", _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, sinks)), bytes_=by)
    add("qwen2 paged_attention decode", _timed(lambda: paged_attention(qd, kd, vd_, dmeta, 0.09)), bytes_=by)
    # ---- rotary + K/V store
    proj = torch.randn(T, (H + 2 * G) * D, device=dev).to(bf)
    pos = torch.arange(T, **i32)
    tab = rope_table(T, D, 1e4, dev)
    cs = rope_cos_sin(T, D, 1e4, dev)
    by = T * (H + 2 * G) * D * 2 * 2.0
    add("rope_vnorm_store", _timed(lambda: rope_vnorm_store(proj, 0, H * D, (H + G) * D, pos, tab, meta.slot_mapping, kc, vc,
                                                            H, G, D, D, D, 1e-5)), bytes_=by)
    add("qwen2 qkv_rope_kvstore", _timed(lambda: qkv_rope_kvstore(proj, None, pos, cs, meta.slot_mapping, kc, vc, H, G, D)),
        bytes_=by)
    # ---- norms at a sublayer boundary
    resid = torch.randn(T, W, device=dev)
    y = torch.randn(T, W, device=dev).to(bf)
    w32, b32, wbf = torch.ones(W, device=dev), torch.zeros(W, device=dev), torch.ones(W, device=dev).to(bf)
    add("dyt_residual (fp32 stream)", _timed(lambda: dyt_residual(resid, y, (0.5, w32, b32), pre=(0.5, w32, b32))),
        bytes_=T * W * (2 + 4 + 4 + 2.0))
    rb = torch.randn(T, W, device=dev).to(bf)
    add("qwen2 add+rmsnorm (bf16 stream)", _timed(lambda: rmsnorm(y, wbf, 1e-6, residual=rb)), bytes_=T * W * 2 * 4.0)
    # ---- GLU
    gu = torch.randn(T, 2 * ff, device=dev).to(bf)
    add("clamped_glu", _timed(lambda: clamped_glu(gu, 7.0)), bytes_=T * ff * 2 * 3.0)
    add("qwen2 silu_mul", _timed(lambda: silu_mul(gu)), bytes_=T * ff * 2 * 3.0)
    # ---- recurrent mixers (no like kernel in Qwen2; fp32 vector flops / state bytes)
    pr = torch.randn(T, 4 * H * D, device=dev).to(bf)
    dec = torch.full((H,), 0.99, device=dev)
    S = torch.zeros(B + 1, H, D, D, device=dev)
    add("decay_attn_scan prefill", _timed(lambda: decay_attention(pr, 0, H * D, 2 * H * D, dec, S, meta, H, D, D), 3, 1),
        flops=4.0 * T * H * D * D, bytes_=T * 3 * H * D * 2.0, peak=VALU_F32)
    prd = torch.randn(B, 4 * H * D, device=dev).to(bf)
    add("decay_attn_scan decode", _timed(lambda: decay_attention(prd, 0, H * D, 2 * H * D, dec, S, dmeta, H, D, D)),
        bytes_=2.0 * B * H * D * D * 4)
    o = torch.randn(T, H * D, device=dev)
    out = torch.empty(T, H * D, device=dev, dtype=bf)
    add("gated_rmsnorm", _timed(lambda: gated_rmsnorm(o, w32[: H * D].contiguous(), pr, 3 * H * D, 1e-5, out)),
        bytes_=T * H * D * (4 + 2 + 2.0))
    gp = torch.randn(T, 3 * W, device=dev).to(bf)
    Sg = torch.zeros(B + 1, W, device=dev)
    add("mingru_scan prefill", _timed(lambda: mingru_scan(gp, 0, W, 2 * W, b32, b32, Sg, meta, W)), bytes_=T * W * 2 * 4.0)
    gpd = torch.randn(B, 3 * W, device=dev).to(bf)
    add("mingru_scan decode", _timed(lambda: mingru_scan(gpd, 0, W, 2 * W, b32, b32, Sg, dmeta, W)),
        bytes_=B * W * (2 * 4 + 8.0))
    return rows


def _namudra_kernel_table(dev, H=28, G=4, D=128, W=3584, T=2048, B=64, ctx=2048, bs=16, win=1024, R=192, r=64, S=2):
    """[(kernel, seconds, bound, fraction of roofline)] for Namudra's kernels and the like kernels of Zofesun."""
    from ..ops.attention import AttnMetadata, sigmoid_window_attention, sink_attention
    from ..ops.elementwise import latent_store, qk_norm_store, rope_table, rope_vnorm_store
    from ..ops.norm import dyt_residual, hyper_mix, rmsnorm_rows
    from ..ops.recurrent import decay_attention, gated_rmsnorm

    bf = torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    rows = []

    def add(name, sec, flops=0.0, bytes_=0.0, peak=MFMA_BF16):
        t_c, t_m = flops / peak, bytes_ / HBM_BPS
        rows.append({"kernel": name, "us": round(sec * 1e6, 1), "bound": "flops" if t_c >= t_m else "bytes",
                     "roofline_fraction": round(max(t_c, t_m) / sec, 4)})

    nb = T // bs
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([0], **i32))
    nbd = ctx // bs
    part_o = torch.empty(8 * B * H * max(D, R), device=dev)
    part_ml = torch.empty(8 * B * H * 2, device=dev)
    dmeta = AttnMetadata(q_start=torch.arange(B + 1, **i32), ctx_len=torch.full((B,), ctx, **i32),
                         block_tables=(torch.arange(B * nbd, **i32) + 1).view(B, nbd), slot_mapping=None, max_q_len=1,
                         num_seqs=B, num_tokens=B, is_decode=True, num_splits=8, split_len=ctx // 8, part_o=part_o,
                         part_ml=part_ml, state_slots=torch.arange(B, **i32))
    # ---- prefill attention, one prompt of T tokens: windowed sigmoid | latent (one kv head, key R + r, value R) | sink
    kc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    vc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    q = torch.randn(T, H, D, device=dev).to(bf)
    gate = torch.randn(T, H * D, device=dev).to(bf)
    pb = torch.zeros(H, device=dev)
    pairs = T * (T + 1) / 2 - (T - win) * (T - win + 1) / 2  # visible (query, key) pairs
    add("sigmoid_window_prefill (window 1024)", _timed(lambda: sigmoid_window_attention(q, kc, vc, meta, 0.09, pb, win, gate=gate)),
        flops=4.0 * pairs * H * D)
    add("zofesun sink_attn_prefill", _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, pb)), flops=4.0 * T * T / 2 * H * D)
    kl = torch.randn(nb + 1, 1, bs, R + r, device=dev).to(bf)
    vl = kl[..., :R]
    ql = torch.randn(T, H, R + r, device=dev).to(bf)
    add("latent attention prefill (sink kernel, no sink)", _timed(lambda: sink_attention(ql, kl, vl, meta, 0.06, None)),
        flops=2.0 * T * T / 2 * H * (2 * R + r))
    # ---- decode attention: B rows of ctx keys
    kd = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    vd_ = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    qd = torch.randn(B, H, D, device=dev).to(bf)
    gd = torch.randn(B, H * D, device=dev).to(bf)
    add("sigmoid_window_decode (window 1024)", _timed(lambda: sigmoid_window_attention(qd, kd, vd_, dmeta, 0.09, pb, win, gate=gd)),
        bytes_=2.0 * B * win * G * D * 2)
    add("zofesun sink_attn_decode", _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, pb)), bytes_=2.0 * B * ctx * G * D * 2)
    kld = torch.randn(B * nbd + 1, 1, bs, R + r, device=dev).to(bf)
    vld = kld[..., :R]
    qld = torch.randn(B, H, R + r, device=dev).to(bf)
    add("latent attention decode (sink kernel, no sink)", _timed(lambda: sink_attention(qld, kld, vld, dmeta, 0.06, None)),
        bytes_=B * ctx * (R + r) * 2.0)
    # ---- projection post-processing + cache stores
    proj = torch.randn(T, (2 * H + G) * D, device=dev).to(bf)
    ones = torch.ones(D, device=dev)
    add("qk_norm_store", _timed(lambda: qk_norm_store(proj, 0, H * D, ones, ones, meta.slot_mapping, kc, vc, H, G, D, 1e-6)),
        bytes_=T * (2 * H + 3 * G) * D * 2.0)
    pos = torch.arange(T, **i32)
    tab = rope_table(T, D, 1e4, dev)
    add("zofesun rope_vnorm_store", _timed(lambda: rope_vnorm_store(proj, 0, H * D, (H + G) * D, pos, tab, meta.slot_mapping, kc, vc,
                                                                    H, G, D, D, D, 1e-5)), bytes_=T * (H + 2 * G) * D * 2 * 2.0)
    ckv = torch.randn(T, R + r, device=dev).to(bf)
    tabr = rope_table(T, r, 1e4, dev)
    wR, wq4 = torch.ones(R, device=dev), torch.ones(W // 4, device=dev)
    add("latent_store", _timed(lambda: latent_store(ckv, wR, pos, tabr, meta.slot_mapping, ql, kl, 1e-6)),
        bytes_=T * ((R + r) * 2 + 2 * H * r) * 2.0)
    cq = torch.randn(T, 2 * (W // 4), device=dev).to(bf)
    add("rmsnorm_rows (query latent)", _timed(lambda: rmsnorm_rows(cq[:, : W // 4], wq4, 1e-6)),
        bytes_=T * (W // 4) * 2 * 2.0)
    # ---- sublayer boundary: S fp32 streams | one fp32 stream
    xs = torch.randn(S, T, W, device=dev)
    y = torch.randn(T, W, device=dev).to(bf)
    mix, oc, ic, w32 = torch.eye(S, device=dev), torch.ones(S, device=dev), torch.ones(S, device=dev) / S, torch.ones(W, device=dev)
    add(f"hyper_mix ({S} fp32 streams)", _timed(lambda: hyper_mix(xs, y, mix, oc, ic, w32, 1e-6)), bytes_=T * W * (2 + 8.0 * S + 2))
    resid = torch.randn(T, W, device=dev)
    b32 = torch.zeros(W, device=dev)
    add("zofesun dyt_residual (one fp32 stream)", _timed(lambda: dyt_residual(resid, y, (0.5, w32, b32), pre=(0.5, w32, b32))),
        bytes_=T * W * (2 + 4 + 4 + 2.0))
    # ---- retention scan (rotary, no activation) | decay scan (SiLU) ; per-head | whole-row gated norm
    pr = torch.randn(T, 4 * H * D, device=dev).to(bf)
    dec = torch.full((H,), 0.99, device=dev)
    St = torch.zeros(B + 1, H, D, D, device=dev)
    add("retention scan prefill", _timed(lambda: decay_attention(pr, 0, H * D, 2 * H * D, dec, St, meta, H, D, D, act=False,
                                                                positions=pos, rope=tab, k_scale=D ** -0.5), 3, 1),
        flops=4.0 * T * H * D * D, bytes_=T * 3 * H * D * 2.0, peak=VALU_F32)
    add("zofesun decay_attn_scan prefill", _timed(lambda: decay_attention(pr, 0, H * D, 2 * H * D, dec, St, meta, H, D, D), 3, 1),
        flops=4.0 * T * H * D * D, bytes_=T * 3 * H * D * 2.0, peak=VALU_F32)
    prd = torch.randn(B, 4 * H * D, device=dev).to(bf)
    posd = torch.full((B,), ctx - 1, **i32)
    add("retention scan decode", _timed(lambda: decay_attention(prd, 0, H * D, 2 * H * D, dec, St, dmeta, H, D, D, act=False,
                                                               positions=posd, rope=tab, k_scale=D ** -0.5)),
        bytes_=2.0 * B * H * D * D * 4)
    add("zofesun decay_attn_scan decode", _timed(lambda: decay_attention(prd, 0, H * D, 2 * H * D, dec, St, dmeta, H, D, D)),
        bytes_=2.0 * B * H * D * D * 4)
    o = torch.randn(T, H * D, device=dev)
    out = torch.empty(T, H * D, device=dev, dtype=bf)
    add("gated_rmsnorm per head, SiLU gate", _timed(lambda: gated_rmsnorm(o, None, pr, 3 * H * D, 1e-6, out, groups=H, gate="silu")),
        bytes_=T * H * D * (4 + 2 + 2.0))
    add("zofesun gated_rmsnorm whole row", _timed(lambda: gated_rmsnorm(o, w32[: H * D].contiguous(), pr, 3 * H * D, 1e-5, out)),
        bytes_=T * H * D * (4 + 2 + 2.0))
    return rows


def _leripel_models(name, dev):
    """Leripel at a bench size: per four layers retention, block-local attention (blocks of 1024), the state-space
    mixer, block-local attention; every layer beside a mixture of 16 experts (4 per token) plus a shared expert whose
    active width equals the dense decoders' feed-forward; beside the Namudra and Qwen2 stacks."""
    from ..models.configs import leripel_config
    from ..models.leripel import LeripelModel

    W, H, G, D, ff, nl, _ = SIZES[name]
    per = (ff // 5) // 64 * 64
    lc = leripel_config(f"leripel-{name}", VOCAB, W, ("rama" * nl)[:nl], heads=H, kv_heads=G, dim=D, chunk=1024,
                        ssm_vdim=64, ssm_state=128, experts=16, top=4, groups=(4, 2), ff=per, shared_ff=ff - 4 * per)
    mk_n, _, mk_q = _namudra_models(name, dev)
    return (lambda: LeripelModel(lc, device=dev, seed=1)), mk_n, mk_q


def _leripel_kernel_table(dev, H=28, G=4, D=128, W=3584, ff=18944, T=2048, B=64, ctx=2048, bs=16, chunk=1024, E=16,
                          top=4, P=64, N=128):
    """[(kernel, seconds, bound, fraction of roofline)] for Leripel's kernels and the like kernels of Namudra."""
    from ..ops.attention import AttnMetadata, sigmoid_window_attention, sink_attention
    from ..ops.elementwise import rope_table, rope_vnorm_store
    from ..ops.linear import linear
    from ..ops.moe import moe_experts, moe_route
    from ..ops.norm import hyper_mix, residual_rmsnorm
    from ..ops.recurrent import causal_conv, decay_attention, gated_rmsnorm, ssm_scan

    bf = torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    rows = []

    def add(name, sec, flops=0.0, bytes_=0.0, peak=MFMA_BF16):
        t_c, t_m = flops / peak, bytes_ / HBM_BPS
        rows.append({"kernel": name, "us": round(sec * 1e6, 1), "bound": "flops" if t_c >= t_m else "bytes",
                     "roofline_fraction": round(max(t_c, t_m) / sec, 4)})

    nb = T // bs
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([0], **i32))
    nbd = ctx // bs
    dmeta = AttnMetadata(q_start=torch.arange(B + 1, **i32), ctx_len=torch.full((B,), ctx, **i32),
                         block_tables=(torch.arange(B * nbd, **i32) + 1).view(B, nbd), slot_mapping=None, max_q_len=1,
                         num_seqs=B, num_tokens=B, is_decode=True, state_slots=torch.arange(B, **i32))
    # ---- attention: blocks of `chunk` positions, temperatures, head gates | sliding window of the same length
    kc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    vc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    q = torch.randn(T, H, D, device=dev).to(bf)
    temp, pb = torch.ones(H, device=dev), torch.zeros(H, device=dev)
    hg = torch.randn(T, H, device=dev).to(bf)
    gate = torch.randn(T, H * D, device=dev).to(bf)
    pairs_c = (T // chunk) * chunk * (chunk + 1) / 2
    pairs_w = T * (T + 1) / 2 - (T - chunk) * (T - chunk + 1) / 2
    add(f"block-local attention prefill (blocks of {chunk})",
        _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, head_scale=temp, head_gate=hg, chunk=chunk)),
        flops=4.0 * pairs_c * H * D)
    add("namudra sigmoid_window_prefill (window 1024)",
        _timed(lambda: sigmoid_window_attention(q, kc, vc, meta, 0.09, pb, chunk, gate=gate)), flops=4.0 * pairs_w * H * D)
    kd = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    vd_ = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    qd = torch.randn(B, H, D, device=dev).to(bf)
    hgd = torch.randn(B, H, device=dev).to(bf)
    gd = torch.randn(B, H * D, device=dev).to(bf)
    dmeta.ctx_len = torch.full((B,), ctx, **i32)  # the last token closes a block: a full block of keys is read
    add(f"block-local attention decode ({chunk} keys)",
        _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, head_scale=temp, head_gate=hgd, chunk=chunk)),
        bytes_=2.0 * B * chunk * G * D * 2)
    add("namudra sigmoid_window_decode (window 1024)",
        _timed(lambda: sigmoid_window_attention(qd, kd, vd_, dmeta, 0.09, pb, chunk, gate=gd)), bytes_=2.0 * B * chunk * G * D * 2)
    # ---- rotary + K/V store
    proj = torch.randn(T, (H + 2 * G) * D + 32, device=dev).to(bf)
    pos = torch.arange(T, **i32)
    tab, tabh = rope_table(T, D, 1e4, dev), rope_table(T, D // 2, 1e4, dev)
    by = T * (H + 2 * G) * D * 2 * 2.0
    add("rope store, adjacent pairs, half the head", _timed(lambda: rope_vnorm_store(
        proj, 0, H * D, (H + G) * D, pos, tabh, meta.slot_mapping, kc, vc, H, G, D, D, D // 2, 1e-5, interleaved=True,
        vnorm=False)), bytes_=by)
    add("zofesun rope_vnorm_store", _timed(lambda: rope_vnorm_store(proj, 0, H * D, (H + G) * D, pos, tab, meta.slot_mapping,
                                                                    kc, vc, H, G, D, D, D, 1e-5)), bytes_=by)
    # ---- layer boundary: mixer + shared + `top` weighted experts into one fp32 residual | two fp32 streams
    x = torch.randn(T, W, device=dev)
    a, b = torch.randn(T, W, device=dev).to(bf), torch.randn(T, W, device=dev).to(bf)
    e = torch.randn(T, top, W, device=dev).to(bf)
    ec, bc, w32 = torch.rand(T, top, device=dev), torch.rand(T, device=dev), torch.ones(W, device=dev)
    add(f"residual_rmsnorm (mixer + shared + {top} experts)", _timed(lambda: residual_rmsnorm(x, a, b, bc, e, ec, w32, 1e-5)),
        bytes_=T * W * (8 + 2.0 * (2 + top) + 2))
    xs = torch.randn(2, T, W, device=dev)
    mix, oc, ic = torch.eye(2, device=dev), torch.ones(2, device=dev), torch.ones(2, device=dev) / 2
    add("namudra hyper_mix (2 fp32 streams)", _timed(lambda: hyper_mix(xs, a, mix, oc, ic, w32, 1e-6)), bytes_=T * W * (2 + 16.0 + 2))
    # ---- state-space mixer | retention scan
    Hs = W // P
    inner, ch = Hs * P, Hs * P + 2 * N
    ld = 2 * inner + 2 * N + Hs
    pj = (torch.randn(T, ld, device=dev) * 0.5).to(bf)
    cw, cb = torch.randn(ch, 4, device=dev) * 0.5, torch.zeros(ch, device=dev)
    cst = torch.zeros(B + 1, 3, ch, device=dev, dtype=bf)
    sst = torch.zeros(B + 1, Hs, N, P, device=dev)
    dtb, alog, dsk = torch.zeros(Hs, device=dev), torch.zeros(Hs, device=dev), torch.ones(Hs, device=dev)
    add("causal_conv prefill (4 taps)", _timed(lambda: causal_conv(pj, inner, cw, cb, cst, meta)), bytes_=T * ch * 2 * 2.0)
    xbc = causal_conv(pj, inner, cw, cb, cst, meta)
    add("ssm_scan prefill", _timed(lambda: ssm_scan(xbc, pj, inner + ch, dtb, alog, dsk, sst, meta, Hs, 1, N, P), 3, 1),
        flops=4.0 * T * Hs * N * P, bytes_=T * ch * 2.0, peak=VALU_F32)
    pr = torch.randn(T, 4 * H * D, device=dev).to(bf)
    dec = torch.full((H,), 0.99, device=dev)
    St = torch.zeros(B + 1, H, D, D, device=dev)
    add("retention scan prefill (no rotary)", _timed(lambda: decay_attention(pr, 0, H * D, 2 * H * D, dec, St, meta, H, D, D, act=False,
                                                                             k_scale=D ** -0.5), 3, 1),
        flops=4.0 * T * H * D * D, bytes_=T * 3 * H * D * 2.0, peak=VALU_F32)
    pjd = (torch.randn(B, ld, device=dev) * 0.5).to(bf)
    add("causal_conv decode", _timed(lambda: causal_conv(pjd, inner, cw, cb, cst, dmeta)), bytes_=B * ch * 2 * (2 + 2 * 3.0))
    xbd = causal_conv(pjd, inner, cw, cb, cst, dmeta)
    add("ssm_scan decode", _timed(lambda: ssm_scan(xbd, pjd, inner + ch, dtb, alog, dsk, sst, dmeta, Hs, 1, N, P)),
        bytes_=2.0 * B * Hs * N * P * 4)
    prd = torch.randn(B, 4 * H * D, device=dev).to(bf)
    add("retention scan decode", _timed(lambda: decay_attention(prd, 0, H * D, 2 * H * D, dec, St, dmeta, H, D, D, act=False,
                                                               k_scale=D ** -0.5)), bytes_=2.0 * B * H * D * D * 4)
    o = torch.randn(T, inner, device=dev)
    out = torch.empty(T, inner, device=dev, dtype=bf)
    add("gated_rmsnorm, gate first, whole row", _timed(lambda: gated_rmsnorm(o, w32[:inner].contiguous(), pj, 0, 1e-5, out, gate="silu",
                                                                             gate_first=True)), bytes_=T * inner * (4 + 2 + 2.0))
    o2 = torch.randn(T, H * D, device=dev)
    out2 = torch.empty(T, H * D, device=dev, dtype=bf)
    add("namudra gated_rmsnorm per head", _timed(lambda: gated_rmsnorm(o2, None, pr, 3 * H * D, 1e-6, out2, groups=H, gate="silu")),
        bytes_=T * H * D * (4 + 2 + 2.0))
    # ---- experts: router, grouped GEMMs | dense GEMMs of the same active width through the engine's linear()
    F = (ff // 5) // 64 * 64
    h = torch.randn(T, W, device=dev).to(bf)
    wr = torch.randn(E + 1, W, device=dev) * 0.05
    add("moe_route (16 experts + gate row)", _timed(lambda: moe_route(h, wr, E, top, 4, 2)), flops=2.0 * T * (E + 1) * W,
        bytes_=T * W * 2.0, peak=VALU_F32)
    ids, _, _ = moe_route(h, wr, E, top, 4, 2)
    wgu = (torch.randn(E, 2 * F, W, device=dev) * 0.02).to(bf)
    wd = (torch.randn(E, W, F, device=dev) * 0.02).to(bf)
    add(f"moe experts prefill ({T} x {top} rows, align + 2 grouped GEMMs)", _timed(lambda: moe_experts(h, ids, wgu, wd)),
        flops=6.0 * T * top * F * W)
    wgd, wdd = (torch.randn(2 * top * F, W, device=dev) * 0.02).to(bf), (torch.randn(W, top * F, device=dev) * 0.02).to(bf)
    hh = torch.randn(T, top * F, device=dev).to(bf)
    add("dense gate|up + down GEMMs of the same active width (linear)",
        _timed(lambda: (linear(h, wgd), linear(hh, wdd))), flops=6.0 * T * top * F * W)
    hd = torch.randn(B, W, device=dev).to(bf)
    idd, _, _ = moe_route(hd, wr, E, top, 4, 2)
    add(f"moe experts decode ({B} x {top} rows)", _timed(lambda: moe_experts(hd, idd, wgu, wd)), bytes_=3.0 * E * F * W * 2)
    hhd = torch.randn(B, top * F, device=dev).to(bf)
    add("dense gate|up + down GEMMs, decode rows (linear)", _timed(lambda: (linear(hd, wgd), linear(hhd, wdd))),
        bytes_=3.0 * top * F * W * 2)
    return rows


def _pubulix_models(name, dev):
    """Pubulix at a bench size: per four layers capped sliding-window attention (window 1024), latent attention with
    its own cache (window 2048), attention again, latent attention over the same cache; every layer with 16
    table-routed experts (4 per token) whose active width equals the dense decoders' feed-forward, an input
    convolution of 4 taps and gated residual branches; beside the Leripel and Qwen2 stacks."""
    from ..models.configs import pubulix_config
    from ..models.pubulix import PubulixModel

    W, H, G, D, ff, nl, _ = SIZES[name]
    pc = pubulix_config(f"pubulix-{name}", VOCAB, W, ("alas" * nl)[:nl], heads=H, kv_heads=G, dim=D, window=1024,
                        lat_heads=H, kv_rank=192, rot_dim=64, lat_window=2048, experts=16, top=4, ff=(ff // 4) // 64 * 64)
    mk_l, _, mk_q = _leripel_models(name, dev)
    return (lambda: PubulixModel(pc, device=dev, seed=1)), mk_l, mk_q


def _pubulix_kernel_table(dev, H=28, G=4, D=128, W=3584, ff=18944, T=2048, B=64, ctx=2048, bs=16, win=1024, lwin=2048,
                          R=192, r=64, E=16, top=4, V=VOCAB):
    """[(kernel, seconds, bound, fraction of roofline)] for Pubulix's kernels and the like kernels of Leripel (attention,
    convolution, boundary, experts) and Namudra (latent attention)."""
    from ..ops.attention import AttnMetadata, sink_attention
    from ..ops.elementwise import latent_rope_store, latent_store, rope_table, tanh_cap_
    from ..ops.linear import linear
    from ..ops.moe import head_project, moe_experts, moe_route, moe_table_route
    from ..ops.norm import residual_rmsnorm
    from ..ops.recurrent import causal_conv

    bf = torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    rows = []

    def add(name, sec, flops=0.0, bytes_=0.0, peak=MFMA_BF16):
        t_c, t_m = flops / peak, bytes_ / HBM_BPS
        rows.append({"kernel": name, "us": round(sec * 1e6, 1), "bound": "flops" if t_c >= t_m else "bytes",
                     "roofline_fraction": round(max(t_c, t_m) / sec, 4)})

    nb = T // bs
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([0], **i32))
    nbd = ctx // bs
    dmeta = AttnMetadata(q_start=torch.arange(B + 1, **i32), ctx_len=torch.full((B,), ctx, **i32),
                         block_tables=(torch.arange(B * nbd, **i32) + 1).view(B, nbd), slot_mapping=None, max_q_len=1,
                         num_seqs=B, num_tokens=B, is_decode=True, state_slots=torch.arange(B, **i32))
    # ---- attention: a window of `win` positions with capped scores | leripel's blocks of the same length
    kc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    vc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    q = torch.randn(T, H, D, device=dev).to(bf)
    temp = torch.ones(H, device=dev)
    hg = torch.randn(T, H, device=dev).to(bf)
    pairs_w = T * (T + 1) / 2 - (T - win) * (T - win + 1) / 2
    pairs_c = (T // win) * win * (win + 1) / 2
    add(f"capped window attention prefill (window {win})",
        _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, window=win, softcap=50.0)), flops=4.0 * pairs_w * H * D)
    add(f"leripel block-local attention prefill (blocks of {win})",
        _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, head_scale=temp, head_gate=hg, chunk=win)),
        flops=4.0 * pairs_c * H * D)
    kd = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    vd_ = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    qd = torch.randn(B, H, D, device=dev).to(bf)
    hgd = torch.randn(B, H, device=dev).to(bf)
    add(f"capped window attention decode ({win} keys)",
        _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, window=win, softcap=50.0)),
        bytes_=2.0 * B * win * G * D * 2)
    add(f"leripel block-local attention decode ({win} keys)",
        _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, head_scale=temp, head_gate=hgd, chunk=win)),
        bytes_=2.0 * B * win * G * D * 2)
    # ---- latent attention: a window and a sink over latent | rotated rows | namudra's causal form on the same rows
    lk = torch.randn(nb + 1, 1, bs, R + r, device=dev).to(bf)
    lq = torch.randn(T, H, R + r, device=dev).to(bf)
    sink = torch.zeros(H, device=dev)
    pairs_l = T * (T + 1) / 2 - max(0, T - lwin) * (max(0, T - lwin) + 1) / 2
    add(f"latent attention prefill (window {lwin}, sink)",
        _timed(lambda: sink_attention(lq, lk, lk[..., :R], meta, 0.06, sink, window=lwin)),
        flops=2.0 * pairs_l * H * (2 * R + r))
    add("namudra latent attention prefill (causal)", _timed(lambda: sink_attention(lq, lk, lk[..., :R], meta, 0.06, None)),
        flops=2.0 * (T * (T + 1) / 2) * H * (2 * R + r))
    lkd = torch.randn(B * nbd + 1, 1, bs, R + r, device=dev).to(bf)
    lqd = torch.randn(B, H, R + r, device=dev).to(bf)
    add(f"latent attention decode ({min(ctx, lwin)} keys, sink)",
        _timed(lambda: sink_attention(lqd, lkd, lkd[..., :R], dmeta, 0.06, sink, window=lwin)),
        bytes_=1.0 * B * min(ctx, lwin) * (R + r) * 2)
    add(f"namudra latent attention decode ({ctx} keys)",
        _timed(lambda: sink_attention(lqd, lkd, lkd[..., :R], dmeta, 0.06, None)), bytes_=1.0 * B * ctx * (R + r) * 2)
    # ---- queries + cache row out of the fused projection | namudra's in-place form
    ld = H * (R + r) + (R + r) + H * D
    proj = torch.randn(T, ld, device=dev).to(bf)
    pos = torch.arange(T, **i32)
    tab = rope_table(T, r, 1e4, dev)
    cw = torch.ones(R, device=dev)
    add("latent_rope_store (queries copied and rotated, cache row)", _timed(lambda: latent_rope_store(
        proj, 0, H * (R + r), cw, pos, tab, meta.slot_mapping, lk, H, 1e-5, interleaved=True)),
        bytes_=T * (H + 1) * (R + r) * 2 * 2.0)
    ckv = torch.randn(T, R + r, device=dev).to(bf)
    add("namudra latent_store (queries rotated in place)", _timed(lambda: latent_store(ckv, cw, pos, tab, meta.slot_mapping,
                                                                                        lq, lk, 1e-5)),
        bytes_=T * (R + r) * 2 * 2.0 + T * H * r * 2 * 2.0)
    # ---- one value matrix per head + gate | one dense GEMM of the same flops through linear()
    o = torch.randn(T, H * R, device=dev).to(bf)
    wuv = (torch.randn(H, D, R, device=dev) * 0.05).to(bf)
    gcol = proj[:, H * (R + r) + (R + r):]
    add(f"head_project prefill ({H} matrices {D} x {R}, gate)", _timed(lambda: head_project(o, wuv, gate=gcol)),
        flops=2.0 * T * H * D * R, bytes_=T * H * (R + 2 * D) * 2.0)
    wdn = (torch.randn(D, H * R, device=dev) * 0.02).to(bf)
    add("dense GEMM of the same flops (linear)", _timed(lambda: linear(o, wdn)), flops=2.0 * T * H * D * R,
        bytes_=T * H * R * 2.0)
    od = torch.randn(B, H * R, device=dev).to(bf)
    gd = torch.randn(B, H * D, device=dev).to(bf)
    add("head_project decode rows", _timed(lambda: head_project(od, wuv, gate=gd)), bytes_=H * D * R * 2.0)
    add("dense GEMM of the same weight bytes, decode rows (linear)", _timed(lambda: linear(od, wdn)), bytes_=H * D * R * 2.0)
    # ---- sublayer boundary: gated branch | leripel's ungated sum of the same operands
    x = torch.randn(T, W, device=dev)
    a = torch.randn(T, W, device=dev).to(bf)
    gt = torch.randn(T, W, device=dev).to(bf)
    e = torch.randn(T, top, W, device=dev).to(bf)
    ec, gb, w32 = torch.rand(T, top, device=dev), torch.zeros(W, device=dev), torch.ones(W, device=dev)
    add("residual_rmsnorm (gated mixer branch)", _timed(lambda: residual_rmsnorm(x, a, w=w32, eps=1e-5, gate=gt, gbias=gb, mult=0.5)),
        bytes_=T * W * (8 + 2.0 * 2 + 2))
    add("leripel residual_rmsnorm (one branch)", _timed(lambda: residual_rmsnorm(x, a, w=w32, eps=1e-5)),
        bytes_=T * W * (8 + 2.0 + 2))
    add(f"residual_rmsnorm (gated sum of {top} experts)",
        _timed(lambda: residual_rmsnorm(x, e=e, ecoef=ec, w=w32, eps=1e-5, gate=gt, gbias=gb, mult=0.5)),
        bytes_=T * W * (8 + 2.0 * (1 + top) + 2))
    add(f"leripel residual_rmsnorm (sum of {top} experts)", _timed(lambda: residual_rmsnorm(x, e=e, ecoef=ec, w=w32, eps=1e-5)),
        bytes_=T * W * (8 + 2.0 * top + 2))
    # ---- input convolution (no activation, input added) | leripel's SiLU form over the same channels
    h = torch.randn(T, W, device=dev).to(bf)
    cwt = torch.randn(W, 4, device=dev) * 0.3
    cst = torch.zeros(B + 1, 3, W, device=dev, dtype=bf)
    add("input convolution prefill (4 taps, h + conv(h))", _timed(lambda: causal_conv(h, 0, cwt, None, cst, meta, act=False, residual=True)),
        bytes_=T * W * 2 * 2.0)
    add("leripel causal_conv prefill (4 taps, SiLU)", _timed(lambda: causal_conv(h, 0, cwt, None, cst, meta)), bytes_=T * W * 2 * 2.0)
    hd = torch.randn(B, W, device=dev).to(bf)
    add("input convolution decode", _timed(lambda: causal_conv(hd, 0, cwt, None, cst, dmeta, act=False, residual=True)),
        bytes_=B * W * 2 * (2 + 2 * 3.0))
    add("leripel causal_conv decode", _timed(lambda: causal_conv(hd, 0, cwt, None, cst, dmeta)), bytes_=B * W * 2 * (2 + 2 * 3.0))
    # ---- experts: table routing, clamped units | leripel's router and SiLU units on the same grouped GEMM
    F = (ff // 4) // 64 * 64
    table = torch.rand(V, E, device=dev).argsort(1)[:, :top].to(torch.int32).contiguous()
    tok = torch.randint(0, V, (T,), device=dev).to(torch.int32)
    wr = torch.randn(E, W, device=dev) * 0.05
    add("moe_table_route", _timed(lambda: moe_table_route(tok, table)), bytes_=T * (4 + top * 12.0))
    add("leripel moe_route (16 experts)", _timed(lambda: moe_route(h, wr, E, top, 4, 2)), flops=2.0 * T * E * W, bytes_=T * W * 2.0,
        peak=VALU_F32)
    ids, _ = moe_table_route(tok, table)
    wgu = (torch.randn(E, 2 * F, W, device=dev) * 0.02).to(bf)
    wd = (torch.randn(E, W, F, device=dev) * 0.02).to(bf)
    add(f"clamped experts prefill ({T} x {top} rows)", _timed(lambda: moe_experts(h, ids, wgu, wd, 7.0, 1.702, 1.0)),
        flops=6.0 * T * top * F * W)
    add(f"leripel SiLU experts prefill ({T} x {top} rows)", _timed(lambda: moe_experts(h, ids, wgu, wd)), flops=6.0 * T * top * F * W)
    idd, _ = moe_table_route(tok[:B].contiguous(), table)
    add(f"clamped experts decode ({B} x {top} rows)", _timed(lambda: moe_experts(hd, idd, wgu, wd, 7.0, 1.702, 1.0)),
        bytes_=3.0 * E * F * W * 2)
    add(f"leripel SiLU experts decode ({B} x {top} rows)", _timed(lambda: moe_experts(hd, idd, wgu, wd)), bytes_=3.0 * E * F * W * 2)
    # ---- logit cap
    lg = torch.randn(B, V, device=dev).to(bf)
    add(f"tanh_cap ({B} x {V} logits)", _timed(lambda: tanh_cap_(lg, 30.0)), bytes_=B * V * 2 * 2.0)
    return rows


def _vudivik_models(name, dev):
    """Vudivik at a bench size: every layer window attention (1024 positions and the first 16) beside a selective scan
    (2 W channels of 16 numbers), feed-forwards in turn dense and 16 experts + 2 identity experts (4 per token), the
    experts' active width equal to the dense one; beside the Leripel and Qwen2 stacks."""
    from ..models.configs import vudivik_config
    from ..models.vudivik import VudivikModel

    W, H, G, D, ff, nl, _ = SIZES[name]
    vc = vudivik_config(f"vudivik-{name}", VOCAB, W, ("dm" * nl)[:nl], heads=H, kv_heads=G, dim=D, ff=ff, window=1024,
                        keep_first=16, experts=16, identity=2, top=4, expert_ff=(ff // 4) // 64 * 64)
    mk_l, _, mk_q = _leripel_models(name, dev)
    return (lambda: VudivikModel(vc, device=dev, seed=1)), mk_l, mk_q


def _vudivik_kernel_table(dev, H=28, G=4, D=128, W=3584, ff=18944, T=2048, B=64, ctx=2048, bs=16, win=1024, keep=16, N=16,
                          E=16, ident=2, top=4):
    """[(kernel, seconds, bound, fraction of roofline)] for Vudivik's kernels and the like kernels of Leripel (scan,
    convolution, boundary, router, experts), Pubulix (window attention, rotary store) and Namudra (normed heads).  The scans are
    priced in vector issue slots (2 flops each): per state number and token a scalar-decay scan needs 2 (the two
    multiply-adds), the per-channel one 8 (two products, the exponential at a quarter of the rate, two multiply-adds)."""
    from ..ops.attention import AttnMetadata, sink_attention
    from ..ops.elementwise import clamped_glu, qk_norm_store, relu2_, rope_table, rope_vnorm_store
    from ..ops.moe import moe_experts, moe_route
    from ..ops.norm import postnorm_residual, residual_rmsnorm
    from ..ops.recurrent import causal_conv, pad_step_matrix, selective_scan, ssm_scan

    bf = torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    rows = []

    def add(name, sec, flops=0.0, bytes_=0.0, peak=MFMA_BF16):
        t_c, t_m = flops / peak, bytes_ / HBM_BPS
        rows.append({"kernel": name, "us": round(sec * 1e6, 1), "bound": "flops" if t_c >= t_m else "bytes",
                     "roofline_fraction": round(max(t_c, t_m) / sec, 4)})

    nb = T // bs
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([0], **i32))
    nbd = ctx // bs
    dmeta = AttnMetadata(q_start=torch.arange(B + 1, **i32), ctx_len=torch.full((B,), ctx, **i32),
                         block_tables=(torch.arange(B * nbd, **i32) + 1).view(B, nbd), slot_mapping=None, max_q_len=1,
                         num_seqs=B, num_tokens=B, is_decode=True, state_slots=torch.arange(B, **i32))
    # ---- attention: a window and the first tokens | the window alone
    kc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    vc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    q = torch.randn(T, H, D, device=dev).to(bf)
    pairs = T * (T + 1) / 2 - (T - win) * (T - win + 1) / 2
    more = sum(min(keep, max(0, i - win + 1)) for i in range(T))
    add(f"window attention with kept tokens prefill (window {win} + {keep})",
        _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, window=win, keep=keep)), flops=4.0 * (pairs + more) * H * D)
    add(f"pubulix window attention prefill (window {win})",
        _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, window=win, softcap=50.0)), flops=4.0 * pairs * H * D)
    kd = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    vd_ = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    qd = torch.randn(B, H, D, device=dev).to(bf)
    add(f"window attention with kept tokens decode ({win} + {keep} keys)",
        _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, window=win, keep=keep)),
        bytes_=2.0 * B * (win + keep) * G * D * 2)
    add(f"pubulix window attention decode ({win} keys)",
        _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, window=win, softcap=50.0)),
        bytes_=2.0 * B * win * G * D * 2)
    # ---- biased, normed, rotated heads + K/V store | normed heads + store, rotated heads + store
    inner, rank = 2 * W, W // 16
    n = (H + 2 * G) * D
    proj = torch.randn(T, n + 2 * inner, device=dev).to(bf)
    pos = torch.arange(T, **i32)
    tab = rope_table(T, D, 5e5, dev)
    bias, qw = torch.zeros(n, device=dev), torch.ones(D, device=dev)
    by = T * n * 2 * 2.0
    add("rope store with biases and head norms", _timed(lambda: rope_vnorm_store(
        proj, 0, H * D, (H + G) * D, pos, tab, meta.slot_mapping, kc, vc, H, G, D, D, D, 1e-6, vnorm=False, bias=bias,
        qw=qw, kw=qw)), bytes_=by)
    add("pubulix rope store", _timed(lambda: rope_vnorm_store(proj, 0, H * D, (H + G) * D, pos, tab, meta.slot_mapping, kc, vc, H, G,
                                                              D, D, D, 1e-6, vnorm=False)), bytes_=by)
    add("namudra qk_norm_store (values are the keys)", _timed(lambda: qk_norm_store(
        proj, 0, H * D, qw, qw, meta.slot_mapping, kc, vc, H, G, D, 1e-6)), bytes_=by)
    # ---- convolution and scan | leripel's over its own channels and state
    cw, cb = torch.randn(inner, 4, device=dev) * 0.5, torch.zeros(inner, device=dev)
    cst = torch.zeros(B + 1, 3, inner, device=dev, dtype=bf)
    Hs, P, Ns = W // 64, 64, 128
    ch = Hs * P + 2 * Ns
    pj = (torch.randn(T, 2 * Hs * P + 2 * Ns + Hs, device=dev) * 0.5).to(bf)
    cws, cbs = torch.randn(ch, 4, device=dev) * 0.5, torch.zeros(ch, device=dev)
    csts = torch.zeros(B + 1, 3, ch, device=dev, dtype=bf)
    add("causal_conv prefill (4 taps)", _timed(lambda: causal_conv(proj, n, cw, cb, cst, meta)), bytes_=T * inner * 2 * 2.0)
    add("leripel causal_conv prefill (4 taps)", _timed(lambda: causal_conv(pj, Hs * P, cws, cbs, csts, meta)), bytes_=T * ch * 2 * 2.0)
    projd = proj[:B].contiguous()
    pjd = pj[:B].contiguous()
    add("causal_conv decode", _timed(lambda: causal_conv(projd, n, cw, cb, cst, dmeta)), bytes_=B * inner * 2 * (2 + 2 * 3.0))
    add("leripel causal_conv decode", _timed(lambda: causal_conv(pjd, Hs * P, cws, cbs, csts, dmeta)), bytes_=B * ch * 2 * (2 + 2 * 3.0))
    xc = causal_conv(proj, n, cw, cb, cst, meta)
    low = torch.randn(T, rank + 2 * N, device=dev).to(bf)
    wdt = pad_step_matrix(torch.randn(inner, rank, device=dev) * rank ** -0.5).to(bf).contiguous()
    dtb, dsk = torch.full((inner,), -3.0, device=dev), torch.ones(inner, device=dev)
    A = -torch.rand(inner, N, device=dev) * N - 0.1
    sst = torch.zeros(B + 1, inner, N, device=dev)
    ssp = torch.zeros(B + 1, Hs, Ns, P, device=dev)
    z1, a1, d1 = torch.zeros(Hs, device=dev), torch.zeros(Hs, device=dev), torch.ones(Hs, device=dev)
    add(f"selective_scan prefill (1 x {T}, step sizes and gate inside)",
        _timed(lambda: selective_scan(xc, low, wdt, rank, dtb, A, dsk, proj, n + inner, sst, meta), 5, 1),
        flops=16.0 * T * inner * N, bytes_=T * inner * 2 * 3.0, peak=VALU_F32)
    xbc = causal_conv(pj, Hs * P, cws, cbs, csts, meta)
    add(f"leripel ssm_scan prefill (1 x {T})", _timed(lambda: ssm_scan(xbc, pj, Hs * P + ch, z1, a1, d1, ssp, meta, Hs, 1, Ns, P), 5, 1),
        flops=4.0 * T * Hs * Ns * P, bytes_=T * ch * 2.0, peak=VALU_F32)
    q4 = torch.arange(5, **i32) * (T // 4)
    m4 = AttnMetadata(q_start=q4, ctx_len=torch.full((4,), T // 4, **i32), block_tables=meta.block_tables.expand(4, -1),
                      slot_mapping=meta.slot_mapping, max_q_len=T // 4, num_seqs=4, num_tokens=T, state_slots=torch.arange(4, **i32))
    add(f"selective_scan prefill (4 x {T // 4})",
        _timed(lambda: selective_scan(xc, low, wdt, rank, dtb, A, dsk, proj, n + inner, sst, m4), 5, 1),
        flops=16.0 * T * inner * N, bytes_=T * inner * 2 * 3.0, peak=VALU_F32)
    add(f"leripel ssm_scan prefill (4 x {T // 4})", _timed(lambda: ssm_scan(xbc, pj, Hs * P + ch, z1, a1, d1, ssp, m4, Hs, 1, Ns, P), 5, 1),
        flops=4.0 * T * Hs * Ns * P, bytes_=T * ch * 2.0, peak=VALU_F32)
    xcd, lowd = xc[:B].contiguous(), low[:B].contiguous()
    add("selective_scan decode (step sizes and gate inside)",
        _timed(lambda: selective_scan(xcd, lowd, wdt, rank, dtb, A, dsk, projd, n + inner, sst, dmeta)),
        bytes_=2.0 * B * inner * N * 4 + 2.0 * inner * rank)
    xbd = xbc[:B].contiguous()
    add("leripel ssm_scan decode", _timed(lambda: ssm_scan(xbd, pjd, Hs * P + ch, z1, a1, d1, ssp, dmeta, Hs, 1, Ns, P)),
        bytes_=2.0 * B * Hs * Ns * P * 4)
    # ---- boundary: normed outputs | leripel's sums of the same operands
    x = torch.randn(T, W, device=dev)
    a, b = torch.randn(T, W, device=dev).to(bf), torch.randn(T, W, device=dev).to(bf)
    e = torch.randn(T, top, W, device=dev).to(bf)
    ec, idw, w32 = torch.rand(T, top, device=dev), torch.rand(T, device=dev), torch.ones(W, device=dev)
    add("postnorm_residual (two mixers)", _timed(lambda: postnorm_residual(x, a, w32, b, w32, 0.5, w=w32, mult=0.7)),
        bytes_=T * W * (8 + 2.0 * 2 + 2))
    add("leripel residual_rmsnorm (two branches)", _timed(lambda: residual_rmsnorm(x, a, b, w=w32)), bytes_=T * W * (8 + 2.0 * 2 + 2))
    add(f"postnorm_residual (sum of {top} experts + identity)",
        _timed(lambda: postnorm_residual(x, e=e, ecoef=ec, idw=idw, w=w32, mult=0.7)), bytes_=T * W * (8 + 2.0 * top + 2))
    add(f"leripel residual_rmsnorm (sum of {top} experts)", _timed(lambda: residual_rmsnorm(x, e=e, ecoef=ec, w=w32)),
        bytes_=T * W * (8 + 2.0 * top + 2))
    xd, ad, bd = x[:B].contiguous(), a[:B].contiguous(), b[:B].contiguous()
    add("postnorm_residual (two mixers), decode rows", _timed(lambda: postnorm_residual(xd, ad, w32, bd, w32, 0.5, w=w32, mult=0.7)),
        bytes_=B * W * (8 + 2.0 * 2 + 2))
    add("leripel residual_rmsnorm (two branches), decode rows", _timed(lambda: residual_rmsnorm(xd, ad, bd, w=w32)),
        bytes_=B * W * (8 + 2.0 * 2 + 2))
    # ---- feed-forward: router, experts, squared relu | leripel's router and SiLU experts, the clamped GLU
    F = (ff // 4) // 64 * 64
    wr = torch.randn(E + ident, W, device=dev) * 0.05
    corr = torch.zeros(E + ident, device=dev)
    add(f"moe_route ({E} + {ident} rows, correction, fp32 input)",
        _timed(lambda: moe_route(x, wr, E + ident, top, corr=corr, identity=ident)), flops=2.0 * T * (E + ident) * W,
        bytes_=T * W * 4.0, peak=VALU_F32)
    add(f"leripel moe_route ({E} rows, groups)", _timed(lambda: moe_route(a, wr[:E].contiguous(), E, top, 4, 2)), flops=2.0 * T * E * W,
        bytes_=T * W * 2.0, peak=VALU_F32)
    ids, _, _ = moe_route(a, wr[:E].contiguous(), E, top)  # (every choice a real expert: the whole product is timed)
    wgu = (torch.randn(E, 2 * F, W, device=dev) * 0.02).to(bf)
    wu = wgu[:, :F].contiguous()
    wd = (torch.randn(E, W, F, device=dev) * 0.02).to(bf)
    add(f"squared-relu experts prefill ({T} x {top} rows)", _timed(lambda: moe_experts(a, ids, wu, wd, unit="relu2")),
        flops=4.0 * T * top * F * W)
    add(f"leripel SiLU experts prefill ({T} x {top} rows)", _timed(lambda: moe_experts(a, ids, wgu, wd)), flops=6.0 * T * top * F * W)
    idd = ids[:B].contiguous()
    add(f"squared-relu experts decode ({B} x {top} rows)", _timed(lambda: moe_experts(ad, idd, wu, wd, unit="relu2")),
        bytes_=2.0 * E * F * W * 2)
    add(f"leripel SiLU experts decode ({B} x {top} rows)", _timed(lambda: moe_experts(ad, idd, wgu, wd)), bytes_=3.0 * E * F * W * 2)
    u = torch.randn(T, ff, device=dev).to(bf)
    gu = torch.randn(T, 2 * ff, device=dev).to(bf)
    add("squared relu (in place)", _timed(lambda: relu2_(u)), bytes_=T * ff * 2 * 2.0)
    add("leripel SiLU-gated unit", _timed(lambda: clamped_glu(gu, None, 1.0, 0.0)), bytes_=T * ff * 2 * 3.0)
    return rows


def _kapanex_models(name, dev):
    """Kapanex at a bench size: delta-rule and window-attention (1024) layers in turn, every layer beside 16 experts (4 per
    token, 2 of 4 groups open) and a shared expert whose active width together equals the dense decoders' feed-forward;
    beside the Leripel and Qwen2 stacks."""
    from ..models.configs import kapanex_config
    from ..models.kapanex import KapanexModel

    W, H, G, D, ff, nl, _ = SIZES[name]
    F = (ff // 5) // 64 * 64
    kc = kapanex_config(f"kapanex-{name}", VOCAB, W, ("da" * nl)[:nl], heads=H, kv_heads=G, dim=D, window=1024, experts=16,
                        top=4, groups=(4, 2), ff=F, shared_ff=ff - 4 * F)
    mk_l, _, mk_q = _leripel_models(name, dev)
    return (lambda: KapanexModel(kc, device=dev, seed=1)), mk_l, mk_q


def _kapanex_kernel_table(dev, H=28, G=4, D=128, W=3584, ff=18944, T=2048, B=64, ctx=2048, bs=16, win=1024, E=16, top=4):
    """[(kernel, seconds, bound, fraction of roofline)] for Kapanex's kernels and the like kernels of Leripel (scan,
    convolution, gated norm, boundary, router, experts), Pubulix (window attention) and Vudivik (normed rotary store).  The
    scans are priced in fp32 vector issue slots (2 flops each) per state number and token: 2 for the scalar-decay scan, 4
    for the delta rule (decay, S^T k, the correction, S^T q), whatever the chunked forms add."""
    from ..ops.attention import AttnMetadata, sink_attention
    from ..ops.elementwise import rope_table, rope_vnorm_store
    from ..ops.moe import moe_experts, moe_route
    from ..ops.norm import residual_layernorm, residual_rmsnorm
    from ..ops.recurrent import causal_conv, gated_delta, gated_rmsnorm, ssm_scan

    bf = torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    rows = []

    def add(name, sec, flops=0.0, bytes_=0.0, peak=MFMA_BF16):
        t_c, t_m = flops / peak, bytes_ / HBM_BPS
        rows.append({"kernel": name, "us": round(sec * 1e6, 1), "bound": "flops" if t_c >= t_m else "bytes",
                     "roofline_fraction": round(max(t_c, t_m) / sec, 4)})

    nb = T // bs
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([0], **i32))
    m4 = AttnMetadata(q_start=torch.arange(5, **i32) * (T // 4), ctx_len=torch.full((4,), T // 4, **i32),
                      block_tables=meta.block_tables.expand(4, -1), slot_mapping=meta.slot_mapping, max_q_len=T // 4,
                      num_seqs=4, num_tokens=T, state_slots=torch.arange(4, **i32))
    nbd = ctx // bs
    dmeta = AttnMetadata(q_start=torch.arange(B + 1, **i32), ctx_len=torch.full((B,), ctx, **i32),
                         block_tables=(torch.arange(B * nbd, **i32) + 1).view(B, nbd), slot_mapping=None, max_q_len=1,
                         num_seqs=B, num_tokens=B, is_decode=True, state_slots=torch.arange(B, **i32))
    # ---- delta rule and gated norm | leripel's scan, gated norm
    vv, C = H * D, 2 * G * D + H * D
    ld = C + vv + 2 * H
    pj = torch.randn(T, ld, device=dev).to(bf)
    cw = torch.randn(C, 4, device=dev) * 0.5
    cst = torch.zeros(B + 1, 3, C, device=dev, dtype=bf)
    sst = torch.zeros(B + 1, H, D, D, device=dev)
    alog, dtb, wn = torch.full((H,), -1.0, device=dev), torch.full((H,), -2.0, device=dev), torch.ones(vv, device=dev)
    xc = causal_conv(pj, 0, cw, None, cst, meta)
    Hs, P, N = W // 64, 64, 128
    ch = Hs * P + 2 * N
    pl = (torch.randn(T, 2 * Hs * P + 2 * N + Hs, device=dev) * 0.5).to(bf)
    cwl, cbl = torch.randn(ch, 4, device=dev) * 0.5, torch.zeros(ch, device=dev)
    cstl = torch.zeros(B + 1, 3, ch, device=dev, dtype=bf)
    sl = torch.zeros(B + 1, Hs, N, P, device=dev)
    z1, a1, d1 = torch.zeros(Hs, device=dev), torch.zeros(Hs, device=dev), torch.ones(Hs, device=dev)
    xl = causal_conv(pl, Hs * P, cwl, cbl, cstl, meta)
    outl = torch.empty(T, Hs * P, device=dev, dtype=bf)
    wl = torch.ones(Hs * P, device=dev)

    def delta(x, p, m):
        return gated_delta(x, p, C + vv, C + vv + H, C, alog, dtb, wn, 1e-6, sst, m, H, G, D, D)

    def ssm(x, p, m, out):
        o = ssm_scan(x, p, Hs * P + ch, z1, a1, d1, sl, m, Hs, 1, N, P)
        return gated_rmsnorm(o, wl, p, 0, 1e-6, out, gate="silu", gate_first=True)

    for m, tag in ((meta, f"1 x {T}"), (m4, f"4 x {T // 4}")):
        add(f"gated_delta prefill ({tag}, gated norm included)", _timed(lambda: delta(xc, pj, m)), flops=8.0 * T * H * D * D,
            bytes_=T * (C + 2 * vv) * 2.0, peak=VALU_F32)
        add(f"leripel ssm_scan + gated_rmsnorm prefill ({tag})", _timed(lambda: ssm(xl, pl, m, outl), 5, 1),
            flops=4.0 * T * Hs * N * P, bytes_=T * (ch + 2 * Hs * P) * 2.0, peak=VALU_F32)
    pjd, pld = pj[:B].contiguous(), pl[:B].contiguous()
    xcd, xld = xc[:B].contiguous(), xl[:B].contiguous()
    add("gated_delta decode (gated norm included)", _timed(lambda: delta(xcd, pjd, dmeta)), bytes_=2.0 * B * H * D * D * 4)
    add("leripel ssm_scan + gated_rmsnorm decode", _timed(lambda: ssm(xld, pld, dmeta, outl[:B])), bytes_=2.0 * B * Hs * N * P * 4)
    add("causal_conv prefill (4 taps)", _timed(lambda: causal_conv(pj, 0, cw, None, cst, meta)), bytes_=T * C * 2 * 2.0)
    add("leripel causal_conv prefill (4 taps)", _timed(lambda: causal_conv(pl, Hs * P, cwl, cbl, cstl, meta)), bytes_=T * ch * 2 * 2.0)
    add("causal_conv decode", _timed(lambda: causal_conv(pjd, 0, cw, None, cst, dmeta)), bytes_=B * C * 2 * (2 + 2 * 3.0))
    add("leripel causal_conv decode", _timed(lambda: causal_conv(pld, Hs * P, cwl, cbl, cstl, dmeta)), bytes_=B * ch * 2 * (2 + 2 * 3.0))
    # ---- window attention | pubulix's (window and score cap)
    kc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    vc = torch.randn(nb + 1, G, bs, D, device=dev).to(bf)
    q = torch.randn(T, H, D, device=dev).to(bf)
    pairs = T * (T + 1) / 2 - (T - win) * (T - win + 1) / 2
    add(f"window attention prefill (window {win})", _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, window=win)),
        flops=4.0 * pairs * H * D)
    add(f"pubulix window attention prefill (window {win})",
        _timed(lambda: sink_attention(q, kc, vc, meta, 0.09, None, window=win, softcap=50.0)), flops=4.0 * pairs * H * D)
    kd = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    vd_ = torch.randn(B * nbd + 1, G, bs, D, device=dev).to(bf)
    qd = torch.randn(B, H, D, device=dev).to(bf)
    by = 2.0 * B * win * G * D * 2
    add(f"window attention decode ({win} keys)", _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, window=win)), bytes_=by)
    add(f"pubulix window attention decode ({win} keys)",
        _timed(lambda: sink_attention(qd, kd, vd_, dmeta, 0.09, None, window=win, softcap=50.0)), bytes_=by)
    # ---- rotated unit heads + K/V store | the same with biases and weights
    n = (H + 2 * G) * D
    proj = torch.randn(T, n, device=dev).to(bf)
    pos = torch.arange(T, **i32)
    tab, tabh = rope_table(T, D, 1e4, dev), rope_table(T, D // 2, 1e4, dev)
    bias, one = torch.zeros(n, device=dev), torch.ones(D, device=dev)
    by = T * n * 2 * 2.0
    add("rope store, unit q / k heads, half the head rotated", _timed(lambda: rope_vnorm_store(
        proj, 0, H * D, (H + G) * D, pos, tabh, meta.slot_mapping, kc, vc, H, G, D, D, D // 2, 1e-6, vnorm=False, qw=one,
        kw=one)), bytes_=by)
    add("vudivik rope store with biases and head norms", _timed(lambda: rope_vnorm_store(
        proj, 0, H * D, (H + G) * D, pos, tab, meta.slot_mapping, kc, vc, H, G, D, D, D, 1e-6, vnorm=False, bias=bias, qw=one,
        kw=one)), bytes_=by)
    # ---- boundary: two layer norms | one RMS norm
    x = torch.randn(T, W, device=dev)
    a, b = torch.randn(T, W, device=dev).to(bf), torch.randn(T, W, device=dev).to(bf)
    e = torch.randn(T, top, W, device=dev).to(bf)
    ec, bc, w32 = torch.rand(T, top, device=dev), torch.rand(T, device=dev), torch.ones(W, device=dev)
    for r, tag in ((T, ""), (B, ", decode rows")):
        xr, args = x[:r].contiguous(), [t[:r].contiguous() for t in (a, b, bc, e, ec)]
        add(f"residual_layernorm (mixer + shared + {top} experts, two norms){tag}",
            _timed(lambda: residual_layernorm(xr, w32, w32, 1e-6, *args)), bytes_=r * W * (8 + 2.0 * (2 + top) + 4))
        add(f"leripel residual_rmsnorm (mixer + shared + {top} experts){tag}",
            _timed(lambda: residual_rmsnorm(xr, *args, w32, 1e-6)), bytes_=r * W * (8 + 2.0 * (2 + top) + 2))
    # ---- router and experts
    F = (ff // 5) // 64 * 64
    wr = torch.randn(E + 1, W, device=dev) * 0.05
    sig = dict(score="sigmoid", group_top=2, scale=2.0)
    ad = a[:B].contiguous()
    for h, r, tag in ((a, T, "prefill"), (ad, B, "decode")):
        add(f"moe_route {tag} (sigmoid, groups by two, {E} + 1 rows)", _timed(lambda: moe_route(h, wr, E, top, 4, 2, **sig)),
            flops=2.0 * r * (E + 1) * W, bytes_=r * W * 2.0, peak=VALU_F32)
        add(f"leripel moe_route {tag} (softmax, groups by one, {E} + 1 rows)", _timed(lambda: moe_route(h, wr, E, top, 4, 2)),
            flops=2.0 * r * (E + 1) * W, bytes_=r * W * 2.0, peak=VALU_F32)
    wgu = (torch.randn(E, 2 * F, W, device=dev) * 0.02).to(bf)
    wd = (torch.randn(E, W, F, device=dev) * 0.02).to(bf)
    ids, _, _ = moe_route(a, wr, E, top, 4, 2, **sig)
    idl, _, _ = moe_route(a, wr, E, top, 4, 2)
    for i, tag in ((ids, ""), (idl, "leripel ")):
        add(f"{tag}experts prefill ({T} x {top} rows)", _timed(lambda: moe_experts(a, i, wgu, wd)), flops=6.0 * T * top * F * W)
        idd = i[:B].contiguous()
        add(f"{tag}experts decode ({B} x {top} rows)", _timed(lambda: moe_experts(ad, idd, wgu, wd)), bytes_=3.0 * E * F * W * 2)
    return rows


def _run_family(names, models, kernel_table) -> dict:
    """A hybrid decoder beside the decoders of equal size: ``names`` (the new one first), ``models`` (size, device) ->
    their constructors in the same order."""
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    sizes = {}
    for name in SIZES:
        makers = dict(zip(names, models(name, dev)))
        cell = {}
        for batch, plen, glen in ((8, 2048, 64), (64, 1024, 64)):
            key = f"B{batch}_P{plen}_G{glen}"
            cell[key] = {k: _engine_numbers(mk, dev, batch, plen, glen) for k, mk in makers.items()}
            print(json.dumps({"size": name, "shape": key, **cell[key]}), flush=True)
        sizes[name] = cell
    kernels = kernel_table(dev)
    for r in kernels:
        print(json.dumps(r), flush=True)
    return {"metric": "_vs_".join(names) + "_tokens_per_s", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
            "sizes": sizes, "kernels": kernels}


FAMILIES = {
    "namudra": (("namudra", "zofesun", "qwen2"), _namudra_models, _namudra_kernel_table),
    "leripel": (("leripel", "namudra", "qwen2"), _leripel_models, _leripel_kernel_table),
    "pubulix": (("pubulix", "leripel", "qwen2"), _pubulix_models, _pubulix_kernel_table),
    "vudivik": (("vudivik", "leripel", "qwen2"), _vudivik_models, _vudivik_kernel_table),
    "kapanex": (("kapanex", "leripel", "qwen2"), _kapanex_models, _kapanex_kernel_table),
}


def run(args) -> dict:
    if getattr(args, "hybrid", None) in FAMILIES:
        return _run_family(*FAMILIES[args.hybrid])
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    sizes = {}
    for name in SIZES:
        mk_z, mk_q = _models(name, dev)
        cell = {}
        for batch, plen, glen in ((8, 2048, 64), (64, 1024, 64)):
            key = f"B{batch}_P{plen}_G{glen}"
            cell[key] = {"zofesun": _engine_numbers(mk_z, dev, batch, plen, glen),
                         "qwen2": _engine_numbers(mk_q, dev, batch, plen, glen)}
            print(json.dumps({"size": name, "shape": key, **cell[key]}), flush=True)
        sizes[name] = cell
    kernels = _kernel_table(dev)
    for r in kernels:
        print(json.dumps(r), flush=True)
    return {"metric": "hybrid_vs_qwen2_tokens_per_s", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
            "sizes": sizes, "kernels": kernels}
