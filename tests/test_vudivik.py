"""Vudivik on the engine, CPU tier: the engine's cache / state / scheduler logic and the ops' host paths against
the float64 oracle (tests/vudivik_oracle.py); the same scenarios run on the HIP kernels in test_vudivik_gpu.py."""
import json

import numpy as np
import pytest
import torch

import vudivik_cases as C
import vudivik_oracle as O
from test_pubulix import _meta

TOL = 3e-5


# ------------------------------------------------------------------------------------------------ mechanisms alone
def boundary_case(device, dtype, tol):
    """The normed output joins the residual: two branches normed apiece, one branch alone, experts' weighted sum with
    identity weights (and pairs of weight 0 whose rows hold NaN), the final norm, the plain copy."""
    from githubrepostorag_amd.ops.norm import postnorm_residual

    g = torch.Generator().manual_seed(1)
    dv = lambda t: None if t is None else t.to(device)
    for T, H, K, mult, eps in ((5, 48, 2, 0.7, 1e-6), (3, 203, 3, 1.0, 1e-2), (2, 4100, 1, 0.25, 1e-5), (4, 9, 2, 2.0, 1e-5),
                               (2, 1300, 4, 0.5, 1e-5)):
        x = torch.randn(T, H, generator=g)
        a, b = (3.0 * torch.randn(T, H, generator=g)).to(dtype), torch.randn(T, H, generator=g).to(dtype)
        wa, wb, w, wn = (1.0 + 0.2 * torch.randn(H, generator=g) for _ in range(4))
        unit = lambda v: O.rms_unit(v, eps)

        def check(xd, h, want, norm, tag):
            assert float((xd.cpu().double() - want).abs().max()) < 3e-5 * max(1.0, float(want.abs().max())), (tag, H)
            hn = unit(want) * wn.double() if norm else want
            assert float((h.cpu().double() - hn).abs().max()) < tol * max(1.0, float(hn.abs().max())), (tag, H)

        kw = dict(w=dv(w), eps=eps, mult=mult, out_dtype=dtype)
        for norm in (False, True):
            xd = x.clone().to(device)
            h = postnorm_residual(xd, dv(a), dv(wa), dv(b), dv(wb), 0.5, wn=dv(wn) if norm else None, **kw)
            y = 0.5 * (unit(a.double()) * wa.double() + unit(b.double()) * wb.double())
            check(xd, h, x.double() + mult * unit(y) * w.double(), norm, "two")
            xd = x.clone().to(device)
            h = postnorm_residual(xd, dv(a), wn=dv(wn) if norm else None, **kw)
            check(xd, h, x.double() + mult * unit(a.double()) * w.double(), norm, "one")
            e = torch.randn(T, K, H, generator=g).to(dtype)
            ec, idw = torch.rand(T, K, generator=g), torch.rand(T, generator=g)
            if K > 1:
                ec[0, 0] = 0.0
            y = (ec.double()[:, :, None] * e.double()).sum(1) + idw.double()[:, None] * x.double()
            if device != "cpu" and K > 1:
                e[0, 0] = float("nan")  # (on the device a pair of weight 0 is not read)
            xd = x.clone().to(device)
            h = postnorm_residual(xd, e=dv(e), ecoef=dv(ec), idw=dv(idw), wn=dv(wn) if norm else None, **kw)
            check(xd, h, x.double() + mult * unit(y) * w.double(), norm, "experts")
            xd = x.clone().to(device)
            h = postnorm_residual(xd, wn=dv(wn) if norm else None, eps=eps, out_dtype=dtype)
            check(xd, h, x.double(), norm, "copy")


def router_case(device, dtype):
    """Chosen by score + correction, weighted by the score alone; identity experts' weights are summed apart.  A
    correction large enough that it decides, tokens on both sides of the few-rows limit."""
    from githubrepostorag_amd.ops.moe import moe_route

    g = torch.Generator().manual_seed(2)
    for E, ident, top, W, T in ((5, 2, 3, 40, 37), (12, 4, 5, 64, 150), (1, 0, 1, 24, 9), (3, 3, 6, 16, 37), (9, 1, 2, 33, 140),
                                (20, 0, 4, 264, 9)):
        h = torch.randn(T, W, generator=g).to(dtype)
        wr = (torch.randn(E + ident, W, generator=g) * 0.7).to(torch.bfloat16).float()
        corr = 0.3 * torch.randn(E + ident, generator=g)
        ids, wts, idw = moe_route(h.to(device), wr.to(device), E + ident, top, corr=corr.to(device), identity=ident)
        want = O.route(h.double(), lambda n: {"router": wr.double(), "correction": corr.double()}[n], {"top": top})
        assert (idw is None) == (ident == 0)
        for t in range(T):
            assert ids[t].tolist() == [e for e, _ in want[t]], (E, t)
            for k, (e, w) in enumerate(want[t]):
                assert abs(float(wts[t, k]) - (float(w) if e < E else 0.0)) < 1e-5
            if ident:
                assert abs(float(idw[t]) - sum(float(w) for e, w in want[t] if e >= E)) < 1e-5
    # the best score loses to a corrected one, and keeps out of the weights
    wr = torch.diag(torch.tensor([2.0, 1.0, 0.5, 0.0]))
    ids, wts, _ = moe_route(torch.ones(1, 4, dtype=dtype, device=device), wr.to(device), 4, 1,
                            corr=torch.tensor([0.0, 0.0, 0.0, 5.0], device=device))
    s = torch.softmax(torch.tensor([2.0, 1.0, 0.5, 0.0]), 0)
    assert ids.tolist() == [[3]] and abs(float(wts[0, 0]) - float(s[3])) < 1e-6


def experts_case(device, dtype, tol):
    """Squared-relu experts; ids past the experts (identity choices) are left out; one expert with no rows."""
    from githubrepostorag_amd.ops.moe import moe_experts

    g = torch.Generator().manual_seed(3)
    for T, W, F, E, top in ((9, 48, 20, 6, 2), (70, 64, 40, 5, 3), (3, 40, 24, 4, 4), (1, 33, 7, 3, 1), (200, 136, 40, 3, 2)):
        h = torch.randn(T, W, generator=g).to(dtype)
        wu = (torch.randn(E, F, W, generator=g) / W ** 0.5).to(dtype)
        wd = (torch.randn(E, W, F, generator=g) / F ** 0.5).to(dtype)
        ids = torch.stack([torch.randperm(E + 2, generator=g)[:top] for _ in range(T)]).to(torch.int32)  # E, E + 1: identity
        if T > 20:
            ids[:, 0] = 1
            ids[ids == 4] = 0
        got = moe_experts(h.to(device), ids.to(device), wu.to(device), wd.to(device), unit="relu2").cpu().double()
        for t in range(T):
            for k in range(top):
                e = int(ids[t, k])
                if e >= E:
                    continue
                want = wd[e].double() @ O.relu2(wu[e].double() @ h[t].double())
                assert float((got[t, k] - want).abs().max()) < tol * max(1.0, float(want.abs().max())), (T, t, k)


def relu2_case(device, dtype):
    from githubrepostorag_amd.ops.elementwise import relu2_

    g = torch.Generator().manual_seed(4)
    for shape in ((3, 40), (5, 7), (1, 1), (33, 264)):
        x = torch.randn(*shape, generator=g).to(dtype)
        got = relu2_(x.clone().to(device)).cpu().double()
        want = O.relu2(x.double())
        assert float((got - want).abs().max()) <= (1e-6 if dtype == torch.float32 else 0.004) * float(want.max().clamp_min(1.0))


def rotary_case(device, dtype, tol):
    """Biased q / k / v out of a fused projection, q / k normed per head before the stretched rotation; values stored as
    projected plus bias.  The frequency table with pairs below, inside and above the blend."""
    from githubrepostorag_amd.models.configs import RopeScaling
    from githubrepostorag_amd.ops.elementwise import rope_table, rope_vnorm_store

    g = torch.Generator().manual_seed(5)
    for H, G, d, vd, rd, base, sc in ((4, 2, 16, 8, 8, 100.0, (4.0, 1.0, 4.0, 40.0)), (3, 1, 72, 70, 72, 1e4, (8.0, 1.0, 4.0, 512.0)),
                                      (2, 2, 10, 24, 0, 1.0, None), (6, 3, 130, 6, 64, 5e3, (2.5, 2.0, 2.5, 300.0)),
                                      (1, 1, 6, 6, 6, 7.0, None)):
        T, bs, eps = 11, 4, 1e-5
        rot = {"dims": rd, "base": base}
        if sc:
            rot["scaling"] = dict(zip(("factor", "low", "high", "original"), sc))
        fr = O.frequencies(rot)
        table = rope_table(2000, rd, base, device, scaling=RopeScaling(*sc) if sc else None) if rd else None
        if sc:  # every kind of pair occurs somewhere in these cases
            p = torch.arange(2000, dtype=torch.float64)
            want = torch.stack([torch.cos(p * f) for f in fr], 1)
            assert float((table[:, :rd // 2].cpu().double() - want).abs().max()) < 1e-6
        n = (H + G) * d + G * vd
        qo, ko, vo = 0, H * d, (H + G) * d
        proj = torch.randn(T, n + 5, generator=g).to(dtype)
        bias = 2.0 * torch.randn(n, generator=g)
        qw, kw = 1.0 + 0.3 * torch.randn(d, generator=g), 1.0 + 0.3 * torch.randn(d, generator=g)
        pos = torch.randint(0, 2000, (T,), generator=g).to(torch.int32)
        slots = torch.randperm(4 * bs, generator=g)[:T].to(torch.int32)
        slots[2] = -1
        kc = torch.zeros(4, G, bs, d, dtype=dtype, device=device)
        vc = torch.zeros(4, G, bs, vd, dtype=dtype, device=device)
        q = rope_vnorm_store(proj.to(device), qo, ko, vo, pos.to(device), table, slots.to(device), kc, vc, H, G, d, vd, rd,
                             eps, vnorm=False, bias=bias.to(device), qw=qw.to(device), kw=kw.to(device))
        x = proj[:, :n].double() + bias.double()
        for t in range(T):
            qn = O.rotate_halves(O.rms_unit(x[t, :H * d].view(H, d), eps) * qw.double(), int(pos[t]), fr)
            assert float((q[t].cpu().double() - qn).abs().max()) < tol * 4, (H, d, t)
            s = int(slots[t])
            if s < 0:
                continue
            kn = O.rotate_halves(O.rms_unit(x[t, ko:vo].view(G, d), eps) * kw.double(), int(pos[t]), fr)
            assert float((kc[s // bs, :, s % bs].cpu().double() - kn).abs().max()) < tol * 4, (H, d, t)
            assert float((vc[s // bs, :, s % bs].cpu().double() - x[t, vo:].view(G, vd)).abs().max()) < tol * 6, (H, d, t)


def scan_case(device, dtype, tol, workgroups=None):
    """Convolution, then the scan, on two sequences at once, cut into steps at different places with stale contents in
    the slots, against one pass of the oracle's loops over each whole sequence.  ``workgroups``: the chip size the
    portions are cut for (None: the default; 1: never cut; 6 and 12: chunks of 256 and 128 for these shapes)."""
    from githubrepostorag_amd.ops import recurrent as R

    g = torch.Generator().manual_seed(6)
    old = R.CHAN_SCAN_WGS
    R.CHAN_SCAN_WGS = workgroups or old
    try:
        for inner, N, rank, taps, lens, steps in (
                (70, 6, 5, 4, (150, 71), ((2, 1), (1, 69), (80, 1), (66, 0), (1, 0))),
                (64, 16, 40, 2, (140, 20), ((139, 1), (1, 2), (0, 17))),
                (33, 37, 3, 1, (90, 66), ((65, 64), (1, 1), (24, 1))),
                (70, 16, 32, 3, (780, 3), ((1, 2), (777, 0), (2, 1)))):
            ld = 8 + 2 * inner + 3
            width = rank + 2 * N
            Wt = {"conv": (torch.randn(inner, taps, generator=g) * 0.5).to(torch.bfloat16).float(),
                  "conv.b": 0.2 * torch.randn(inner, generator=g), "x": torch.randn(width, inner, generator=g) / inner ** 0.5,
                  "dt": torch.randn(inner, rank, generator=g) / rank ** 0.5, "dt.b": torch.randn(inner, generator=g) - 2.0,
                  "A": -torch.exp(torch.rand(inner, N, generator=g) * 4.0 - 3.0), "D": 1 + 0.3 * torch.randn(inner, generator=g)}
            Wt["x"], Wt["dt"] = Wt["x"].to(dtype), Wt["dt"].to(dtype)
            seqs = [torch.randn(n, ld, generator=g).to(dtype) for n in lens]
            lows = [torch.randn(n, -(-width // 8) * 8, generator=g).to(dtype) for n in lens]  # (the pad holds numbers too)
            want = []
            for s, lo in zip(seqs, lows):
                xc = O.short_conv(s[:, 8:8 + inner].double(), Wt["conv"].double(), Wt["conv.b"].double())
                if dtype != torch.float32:
                    xc = xc.to(dtype).double()  # the convolution's output is stored in the activation type
                dt = O.softplus(lo[:, :rank].double() @ Wt["dt"].double().T + Wt["dt.b"].double())
                y = O.selective_scan(xc, dt, Wt["A"].double(), lo[:, rank:rank + N].double(), lo[:, rank + N:width].double(),
                                     Wt["D"].double())
                want.append(y * O.silu(s[:, 8 + inner:8 + 2 * inner].double()))
            cstate = torch.randn(3, taps - 1, inner, generator=g).to(dtype).to(device)  # stale
            sstate = torch.randn(3, inner, N, generator=g).to(device)
            dv = lambda n: Wt[n].to(device)
            wdt = R.pad_step_matrix(dv("dt")).contiguous()
            got, cur = [[], []], [0, 0]
            for step in steps:
                rows, lrows, ls, cs, sl, who = [], [], [], [], [], []
                for i, n in enumerate(step):
                    if n:
                        rows.append(seqs[i][cur[i]:cur[i] + n])
                        lrows.append(lows[i][cur[i]:cur[i] + n])
                        cur[i] += n
                        ls.append(n); cs.append(cur[i]); sl.append(2 - i); who.append(i)
                proj, low = torch.cat(rows, 0).to(device), torch.cat(lrows, 0).to(device)
                meta = _meta(device, ls, cs, sl, decode=max(ls) == 1)
                xc = R.causal_conv(proj, 8, dv("conv"), dv("conv.b"), cstate, meta)
                y = R.selective_scan(xc, low, wdt, rank, dv("dt.b"), dv("A"), dv("D"), proj, 8 + inner, sstate, meta)
                o = 0
                for i, n in zip(who, ls):
                    got[i].append(y[o:o + n].cpu().double())
                    o += n
            for i in range(2):
                assert cur[i] == lens[i]
                err = float((torch.cat(got[i], 0) - want[i]).abs().max() / want[i].abs().max())
                assert err < tol, (inner, N, i, err)
    finally:
        R.CHAN_SCAN_WGS = old


def test_boundary_alone():
    boundary_case("cpu", torch.float32, 1e-5)


def test_router_alone():
    router_case("cpu", torch.float32)


def test_experts_alone():
    experts_case("cpu", torch.float32, 1e-5)


def test_squared_relu_alone():
    relu2_case("cpu", torch.float32)


def test_rotary_alone():
    rotary_case("cpu", torch.float32, 1e-5)


def test_scan_alone():
    scan_case("cpu", torch.float32, 1e-5)


def test_scan_chunk_lengths():
    from githubrepostorag_amd.ops.recurrent import _chan_chunk

    assert _chan_chunk(1, 1, 4096) == 0 and _chan_chunk(64, 64, 4096) == 0  # decode rows, short portions
    assert _chan_chunk(1, 4096, 3072) == 128 and _chan_chunk(1, 8192, 7168) == 256  # one long prompt
    assert _chan_chunk(16, 1024, 3072) == 0  # enough sequences to fill the chip
    assert _chan_chunk(1, 100, 64) == 64


def test_window_edges_in_prompts_and_decoding():
    C.case_window_edges("cpu", 1e-5)
    C.case_window_edges("cpu", 1e-5, bs=4, windows=(3, 4, 30))


# ------------------------------------------------------------------------------------------------ the engine
def test_whole_prompt_and_layer_taps():
    C.case_whole_and_layers("cpu", TOL)


@pytest.mark.parametrize("mlp", [O.DENSE, O.MOE, None])
def test_single_layer_models(mlp):
    C.case_single_layer("cpu", TOL, mlp, n=33)


@pytest.mark.parametrize("branch", ["left", "right"])
def test_one_branch_models(branch):
    C.case_one_branch("cpu", TOL, branch)


def test_shared_tensors():
    C.case_shared_tensors("cpu", TOL)


def test_prefill_against_decode():
    C.case_prefill_vs_decode("cpu", TOL, n=44)


def test_portions():
    C.case_portions("cpu", TOL)


def test_unequal_batches():
    C.case_batches("cpu", TOL)


def test_pages_and_slots_used_again():
    C.case_reuse("cpu", TOL)


def test_other_sizes():
    C.case_other_sizes("cpu", TOL)


def test_unlike_layers():
    C.case_mixed_layers("cpu", TOL)


def test_first_tokens():
    C.case_first_tokens("cpu", TOL)


def test_long_decode():
    C.case_long_decode("cpu", TOL)


def test_sharp_softmax_picks_far_keys():
    C.case_sharp_far_keys("cpu", 2e-4)


def test_greedy_generation_through_the_scheduler():
    C.case_generate("cpu")
    C.case_generate("cpu", mixed=True, max_batched=16)


def test_config_round_trip_and_registry(tmp_path):
    from safetensors.torch import save_file

    from githubrepostorag_amd.models import load_decoder
    from githubrepostorag_amd.models.configs import (config_from_dir, decoder_config, vudivik_config_from_dict,
                                                     vudivik_config_to_dict)
    from githubrepostorag_amd.models.vudivik import init_state_dict

    cfg = O.make_config(shared={2: 1}, mlps=(O.DENSE, O.MOE, O.MOE))
    assert vudivik_config_to_dict(vudivik_config_from_dict(cfg)) == cfg
    tiny = decoder_config("vudivik-tiny")
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(vudivik_config_to_dict(tiny)))
    sd = init_state_dict(tiny, seed=1)
    save_file({k: v.contiguous() for k, v in sd.items()}, str(d / "model.safetensors"))
    assert config_from_dir(d).layers == tiny.layers
    model = load_decoder(d, device="cpu", dtype=torch.float32)
    assert type(model).__name__ == "VudivikModel" and len(model.runs) == 4
    assert tiny.param_count() == sum(v.numel() for v in sd.values())
    # a tensor of the wrong shape is refused by name
    bad = dict(sd)
    bad["l1.mix.right.dt"] = bad["l1.mix.right.dt"][:-1]
    with pytest.raises(ValueError, match="l1.mix.right.dt"):
        type(model)(tiny, device="cpu", dtype=torch.float32, state_dict=bad)
    # a layer that differs from the one whose tensors it uses, a circle, and a missing layer are refused
    for change in (lambda c: c["layers"][2]["mixer"]["left"].update(scale=9.0), lambda c: c["layers"][1].update(weights_of=2),
                   lambda c: c["layers"][2].update(weights_of=7)):
        wrong = json.loads(json.dumps(cfg))
        change(wrong)
        with pytest.raises(ValueError, match="layer"):
            vudivik_config_from_dict(wrong)


def test_trace_replay(tmp_path):
    """The replay command on a saved checkpoint: portions, a request that sits out a step, slots used again."""
    import io

    from safetensors.torch import save_file

    from githubrepostorag_amd.engine.trace import run_trace

    cfg = O.make_config()
    sd = O.make_weights(cfg, seed=31)
    d = tmp_path / "m"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(d / "model.safetensors"))
    a, b = C.tokens(cfg, 30, 1), C.tokens(cfg, 12, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:11], "want": []}, {"id": "a", "tokens": a[17:18], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[18:], "want": [11]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b[11:], "want": [0]}], "end": ["b"]}]
    log = io.StringIO()
    out = tmp_path / "o"
    assert run_trace(str(d), "float32", str(out), 128, device="cpu", lines=[json.dumps(s) for s in steps], log=log) == 0
    assert log.getvalue().split() == ["done", "0", "done", "1", "done", "2", "done", "3"]
    wa, wb = O.forward(cfg, sd, a), O.forward(cfg, sd, b)
    rd = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
    assert C.rel_err(rd(0), wa[[0, 16]]) < TOL and C.rel_err(rd(1), wa[[17]]) < TOL
    assert C.rel_err(rd(2), wa[[29]]) < TOL and C.rel_err(rd(3), wb[[11]]) < TOL
