"""Kapanex on the engine, CPU tier: the engine's cache / state / scheduler logic and the ops' host paths against
the float64 oracle (tests/kapanex_oracle.py); the same scenarios run on the HIP kernels in test_kapanex_gpu.py."""
import json

import numpy as np
import pytest
import torch

import kapanex_cases as C
import kapanex_oracle as O
from test_pubulix import _meta

TOL = 3e-5


# ------------------------------------------------------------------------------------------------ mechanisms alone
def boundary_case(device, dtype, tol):
    """Mixer, gated shared expert and weighted experts join the residual, whose two layer norms come out together; rows
    far from zero (where a variance from squares would drown), rows past the register path, only one norm, no addend."""
    from githubrepostorag_amd.ops.norm import residual_layernorm

    g = torch.Generator().manual_seed(1)
    dv = lambda t: None if t is None else t.to(device)
    for T, H, K, off, eps in ((5, 48, 2, 0.0, 1e-6), (3, 203, 3, 5.0, 1e-2), (2, 4100, 1, 300.0, 1e-5), (4, 9, 0, 0.0, 1e-5),
                              (2, 5000, 0, 40.0, 1e-5), (3, 1300, 4, -7.0, 1e-5), (2, 5, 1, 0.0, 1e-5)):
        x = off + torch.randn(T, H, generator=g)
        a, b = torch.randn(T, H, generator=g).to(dtype), torch.randn(T, H, generator=g).to(dtype)
        e = torch.randn(T, K, H, generator=g).to(dtype) if K else None
        ec, bc = torch.rand(T, K, generator=g) if K else None, torch.rand(T, generator=g)
        w, w2 = 1.0 + 0.2 * torch.randn(H, generator=g), 1.0 + 0.2 * torch.randn(H, generator=g)
        full = x.double() + a.double() + b.double() * bc.double()[:, None]
        if K:
            full = full + (ec.double()[:, :, None] * e.double()).sum(1)
        for want, kw in ((full, dict(a=dv(a), b=dv(b), bcoef=dv(bc), e=dv(e), ecoef=dv(ec))),
                         (x.double() + a.double(), dict(a=dv(a))), (x.double(), {})):
            for both in (True, False):
                xd = x.clone().to(device)
                h1, h2 = residual_layernorm(xd, dv(w), dv(w2) if both else None, eps, out_dtype=dtype, **kw)
                assert float((xd.cpu().double() - want).abs().max()) < 1e-6 * max(10.0, abs(off))
                assert (h2 is not None) == both
                for h, ww in ((h1, w), (h2, w2)):
                    if h is not None:
                        n = O.layer_norm(want, ww.double(), eps)
                        assert float((h.cpu().double() - n).abs().max()) < (tol + 1e-6 * abs(off)) * float(n.abs().max()), H


def router_case(device, dtype):
    """Sigmoid scores, groups worth their two best, weights that sum to a constant; groups of one expert, one group,
    tokens on both sides of the few-rows limit; a group with the single best expert that two good ones beat."""
    from githubrepostorag_amd.ops.moe import moe_route

    g = torch.Generator().manual_seed(2)
    for E, top, groups, keep, W, T, scale in ((32, 4, 8, 4, 40, 140, 1.0), (100, 16, 4, 2, 40, 140, 1.0), (32, 3, 1, 1, 40, 9, 2.0), (6, 2, 3, 2, 40, 37, 1.7), (20, 4, 5, 3, 64, 150, 2.2), (8, 8, 1, 1, 24, 37, 1.0),
                                              (9, 1, 9, 1, 16, 37, 0.3), (15, 4, 5, 5, 33, 131, 1.0), (24, 5, 6, 2, 264, 9, 3.0),
                                              (140, 6, 70, 5, 64, 20, 2.0), (1, 1, 1, 1, 24, 140, 4.0)):
        h = torch.randn(T, W, generator=g).to(dtype)
        wr = (torch.randn(E + 1, W, generator=g) * 2.0 / W ** 0.5).to(torch.bfloat16).float()
        ids, wts, gate = moe_route(h.to(device), wr.to(device), E, top, groups, keep, score="sigmoid", group_top=2, scale=scale)
        r = {"experts": E, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}}
        want = O.route(h.double(), lambda n: {"router": wr[:E].double()}[n], r)
        for t in range(T):
            assert ids[t].tolist() == [e for e, _ in want[t]], (E, t)
            for k, (_, w) in enumerate(want[t]):
                assert abs(float(wts[t, k]) - float(w)) < 1e-5 * scale
        z = h.double() @ wr[E].double()
        assert float((gate.cpu().double() - torch.sigmoid(z)).abs().max()) < 1e-5
    wr = torch.diag(torch.tensor([2.0, -3.0, 1.0, 1.1])).to(device)
    h = torch.ones(1, 4, dtype=dtype, device=device)
    ids, wts, _ = moe_route(h, wr, 4, 2, 2, 1, score="sigmoid", group_top=2, scale=1.0)
    assert ids.tolist() == [[3, 2]] and abs(float(wts.sum()) - 1.0) < 1e-6
    ids, _, _ = moe_route(h, wr, 4, 2, 2, 1, score="sigmoid", group_top=1, scale=1.0)
    assert ids.tolist() == [[0, 1]]


def rotary_case(device, dtype, tol):
    """q and k rotated, then divided by their root mean square; v as projected."""
    from githubrepostorag_amd.ops.elementwise import rope_table, rope_vnorm_store

    g = torch.Generator().manual_seed(5)
    for H, G, d, vd, rd, base, eps in ((4, 2, 16, 8, 8, 100.0, 1e-5), (3, 1, 48, 70, 48, 1e4, 0.5), (2, 2, 10, 24, 0, 1.0, 1e-5),
                                       (6, 3, 130, 6, 64, 5e3, 1e-5), (8, 2, 128, 64, 64, 1e6, 1e-2)):
        T, bs = 11, 4
        table = rope_table(2000, rd, base, device) if rd else None
        n = (H + G) * d + G * vd
        proj = torch.randn(T, n + 8 + -n % 8, generator=g).to(dtype)
        pos = torch.randint(0, 2000, (T,), generator=g).to(torch.int32)
        slots = torch.randperm(4 * bs, generator=g)[:T].to(torch.int32)
        kc, vc = (torch.zeros(4, G, bs, s, dtype=dtype, device=device) for s in (d, vd))
        ones = torch.ones(d, device=device)
        q = rope_vnorm_store(proj.to(device), 0, H * d, (H + G) * d, pos.to(device), table, slots.to(device), kc, vc, H, G, d,
                             vd, rd, eps, vnorm=False, qw=ones, kw=ones)
        for t in range(T):
            row = proj[t].double()
            turn = lambda x: O.rms_unit(O.rotate_halves(x, int(pos[t]), rd, base), eps)
            b, o = int(slots[t]) // bs, int(slots[t]) % bs
            for got, want in ((q[t], turn(row[:H * d].view(H, d))), (kc[b, :, o], turn(row[H * d:(H + G) * d].view(G, d))),
                              (vc[b, :, o], row[(H + G) * d:n].view(G, vd))):
                assert float((got.cpu().double() - want).abs().max()) < tol * max(1.0, float(want.abs().max())), (H, d, t)


DELTA_SIZES = [  # H, G, d, vd, taps
    (6, 3, 12, 20, 4), (5, 1, 64, 96, 3), (2, 2, 33, 7, 2), (3, 3, 130, 48, 1), (2, 1, 256, 256, 4), (4, 2, 128, 128, 4),
    (1, 1, 1, 1, 2), (2, 1, 40, 255, 5),
]


def delta_case(device, dtype, tol, sizes=None, crafted=False):
    """Convolution, delta rule and gated norm alone: two sequences in one step, cut at different places, in slots that
    hold another sequence's leftovers; portions that end on, before and behind a chunk (64) and a block (16), then
    single tokens.  ``crafted``: unit decays and steps near 1, keys that repeat, one write at the start that only the last
    token asks for."""
    from githubrepostorag_amd.ops.recurrent import causal_conv, gated_delta

    for n, (H, G, d, vd, taps) in enumerate(sizes or DELTA_SIZES):
        g = torch.Generator().manual_seed(30 + n)
        eps, L = 1e-5, (150, 131)
        C0, vv = 2 * G * d + H * vd, H * vd
        ld = C0 + vv + 2 * H + 3
        projs = [torch.randn(t, ld, generator=g).to(dtype) for t in L]
        alog, dtb = torch.rand(H, generator=g) * 2.0 - (1.5 if n % 2 else 5.0), torch.randn(H, generator=g) - 1.0
        wn, cw = 1.0 + 0.3 * torch.randn(vd, generator=g), 0.6 * torch.randn(C0, taps, generator=g)
        if crafted:
            cw = torch.zeros(C0, taps)
            cw[:, -1] = 1.0  # only the token itself
            alog = torch.full((H,), -12.0)
            for p in projs:
                p[:, C0 + vv:C0 + vv + H] = 6.0  # steps near 1
                q, k = p[:, :G * d].view(-1, G, d), p[:, G * d:2 * G * d].view(-1, G, d)
                q[:], k[:] = -3.0, -3.0
                k[1:, :, 1:] += 4.0 * torch.randn(len(p) - 1, G, d - 1, generator=g).abs().to(dtype).clamp_max(3.0)
                k[0, :, 0], q[-1, :, 0] = 9.0, 9.0  # the first token's key, asked for by the last
                k[40:60] = k[40:41]  # the same key over and over, across a block border
        w = wn.repeat(H)
        state = torch.randn(3, H, d, vd, generator=g).to(device)
        conv = torch.randn(3, taps - 1, C0, generator=g).to(dtype).to(device)
        want, last = [], []
        for p in projs:  # (the convolution is rounded to the activation type, as the op stores it)
            xc = O.short_conv(p[:, :C0].double(), cw.double()).to(dtype).double()
            q, k = (O.unit(xc[:, i * G * d:(i + 1) * G * d].view(-1, G, d)).repeat_interleave(H // G, dim=1) for i in (0, 1))
            z = p.double()
            dec = torch.exp(-torch.exp(alog.double()) * O.softplus(z[:, C0 + vv + H:C0 + vv + 2 * H] + dtb.double()))
            o, S = O.delta_rule(q * d ** -0.5, k, xc[:, 2 * G * d:].view(-1, H, vd), dec,
                                torch.sigmoid(z[:, C0 + vv:C0 + vv + H]))
            want.append((O.rms_unit(o, eps) * wn.double() * O.silu(z[:, C0:C0 + vv].view(-1, H, vd))).reshape(-1, vv))
            last.append(S)
        dv = lambda t: t.to(device)
        cur, got = [0, 0], [[], []]
        for cuts in ((63, 2), (3, 64), (65, 50), (1, 1), (1, 1), (15, 12), (1, 1), (1, 0)):
            seqs = [s for s in (0, 1) if cuts[s]]
            m = _meta(device, [cuts[s] for s in seqs], [cur[s] + cuts[s] for s in seqs], [2 - s for s in seqs],
                      decode=max(cuts) == 1)
            p = dv(torch.cat([projs[s][cur[s]:cur[s] + cuts[s]] for s in seqs]))
            xc = causal_conv(p, 0, dv(cw), None, conv, m)
            y = gated_delta(xc, p, C0 + vv, C0 + vv + H, C0, dv(alog), dv(dtb), dv(w), eps, state, m, H, G, d, vd)
            at = 0
            for s in seqs:
                got[s].append(y[at:at + cuts[s]].cpu().double())
                at += cuts[s]
                cur[s] += cuts[s]
        assert cur == [150, 131]
        for s in (0, 1):
            a = torch.cat(got[s])
            # (a read-out of almost nothing is blown up by its norm, so rows are judged by their own error)
            err = (a - want[s]).pow(2).mean(1).sqrt() / want[s].pow(2).mean(1).sqrt()
            assert float(err.max()) < (20 * tol if vd == 1 else tol), (n, s, int(err.argmax()), float(err.max()))
            dS = (state[2 - s].cpu().double() - last[s]).abs().max() / last[s].abs().max()
            assert float(dS) < tol, (n, s, float(dS))


def test_boundary_alone():
    boundary_case("cpu", torch.float32, 1e-5)


def test_router_alone():
    router_case("cpu", torch.float32)


def test_rotary_alone():
    rotary_case("cpu", torch.float32, 1e-5)


def test_delta_rule_alone():
    delta_case("cpu", torch.float32, 1e-4, O_SMALL)
    delta_case("cpu", torch.float32, 2e-3, O_SMALL[:1], crafted=True)


O_SMALL = [DELTA_SIZES[0], DELTA_SIZES[2], DELTA_SIZES[6]]


def test_window_edges_in_prompts_and_decoding():
    C.case_window_edges("cpu", 1e-5)
    C.case_window_edges("cpu", 1e-5, bs=4, windows=(3, 4, 30))


# ------------------------------------------------------------------------------------------------ the engine
def test_whole_prompt_and_layer_taps():
    C.case_whole_and_layers("cpu", TOL)


@pytest.mark.parametrize("kind", [O.DELTA, O.ATT])
@pytest.mark.parametrize("moe", [True, False])
def test_single_layer_models(kind, moe):
    C.case_single_layer("cpu", TOL, kind, moe, n=40)


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
    from githubrepostorag_amd.models.configs import (config_from_dir, decoder_config, kapanex_config_from_dict,
                                                     kapanex_config_to_dict)
    from githubrepostorag_amd.models.kapanex import init_state_dict

    cfg = O.make_config(shared={2: 0}, moe=(True, False, True))
    assert kapanex_config_to_dict(kapanex_config_from_dict(cfg)) == cfg
    tiny = decoder_config("kapanex-tiny")
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(kapanex_config_to_dict(tiny)))
    sd = init_state_dict(tiny, seed=1)
    save_file({k: v.contiguous() for k, v in sd.items()}, str(d / "model.safetensors"))
    assert config_from_dir(d).layers == tiny.layers and config_from_dir(d).embed_scale == tiny.embed_scale
    model = load_decoder(d, device="cpu", dtype=torch.float32)
    assert type(model).__name__ == "KapanexModel" and len(model.runs) == 4
    assert tiny.param_count() == sum(v.numel() for v in sd.values())
    # a tensor of the wrong shape and a missing one are refused by name
    bad = dict(sd)
    bad["l0.mix.k.conv"] = bad["l0.mix.k.conv"][:, :-1]
    with pytest.raises(ValueError, match="l0.mix.k.conv"):
        type(model)(tiny, device="cpu", dtype=torch.float32, state_dict=bad)
    del bad["l0.mix.k.conv"]
    with pytest.raises(KeyError, match="l0.mix.k.conv"):
        type(model)(tiny, device="cpu", dtype=torch.float32, state_dict=bad)
    # a layer that differs from the one whose tensors it uses, a circle, a missing layer and bad sizes are refused
    for change in (lambda c: c["layers"][2]["mixer"].update(vdim=9), lambda c: c["layers"][0].update(weights_of=2),
                   lambda c: c["layers"][2].update(weights_of=7)):
        wrong = json.loads(json.dumps(cfg))
        change(wrong)
        with pytest.raises(ValueError, match="layer"):
            kapanex_config_from_dict(wrong)
    for change in (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
                   lambda c: c["layers"][0]["mlp"]["router"].update(top=5), lambda c: c["layers"][1].update(type="other")):
        wrong = json.loads(json.dumps(dict(cfg, layers=cfg["layers"][:2])))
        change(wrong)
        with pytest.raises(ValueError):
            kapanex_config_from_dict(wrong)


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
