"""Scenarios that compare the engine serving a Kapanex model (kernels, paged cache, state slots, scheduler) with
the plain float64 oracle of kapanex_oracle.py.  Every scenario takes the device: the CPU tier runs the ops' host
paths, the GPU tier the HIP kernels, through the same engine code."""
from __future__ import annotations

import numpy as np
import torch

import kapanex_oracle as O
from kapanex_oracle import ATT, DELTA
from leripel_cases import feed_in_portions, near_ties, rel_err  # noqa: F401  (helpers that know no design)


def build(cfg_dict, sd, device, dtype=torch.float32, slots=4, pool_tokens=512, block_size=16, graphs=False,
          max_batched=4096, mixed=False, window=1):
    from githubrepostorag_amd.engine.llm_engine import EngineConfig, LLMEngine
    from githubrepostorag_amd.models import build_decoder
    from githubrepostorag_amd.models.configs import kapanex_config_from_dict

    model = build_decoder(kapanex_config_from_dict(cfg_dict), device=device, dtype=dtype, state_dict=sd)
    eng = LLMEngine(model, None, EngineConfig(max_num_seqs=slots, max_model_len=max(pool_tokens, 64),
                                              block_size=block_size, num_blocks=pool_tokens // block_size + 1,
                                              use_cuda_graph=graphs, max_num_batched_tokens=max_batched,
                                              mixed_batches=mixed, decode_window=window))
    return model, eng


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(7000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def slow_decay(sd):
    """Decays near 1: the delta rule's state remembers the whole sequence, so a lost or foreign one shows."""
    return {k: v - 4.0 if k.endswith("A_log") else v for k, v in sd.items()}


def case_whole_and_layers(device, tol, dtype=torch.float32, **cfg_kw):
    cfg = O.make_config(**cfg_kw)
    sd = O.make_weights(cfg, seed=3)
    toks = tokens(cfg, 37, 0)
    want, taps = O.logits_and_taps(cfg, sd, toks)
    model, eng = build(cfg, sd, device, dtype)
    assert rel_err(feed_in_portions(eng, "a", toks, [len(toks)]), want) < tol
    # the residual after every layer, through the model's own step (one sequence, fresh cache / state)
    from githubrepostorag_amd.ops.attention import AttnMetadata

    T, bs = len(toks), 16
    nb = -(-T // bs)
    i32 = dict(dtype=torch.int32, device=model.device)
    meta = AttnMetadata(q_start=torch.tensor([0, T], **i32), ctx_len=torch.tensor([T], **i32),
                        block_tables=(torch.arange(nb, **i32) + 1).view(1, nb), slot_mapping=torch.arange(T, **i32) + bs,
                        max_q_len=T, num_seqs=1, num_tokens=T, state_slots=torch.tensor([1], **i32))
    mine = []
    model.forward(torch.tensor(toks, **i32), torch.arange(T, **i32), meta, model.allocate_kv_cache(nb + 1, bs),
                  state=model.allocate_state(2), taps=mine)
    assert len(mine) == taps.shape[0]
    for r, (a, b) in enumerate(zip(mine, taps)):
        err = float((a.double().cpu() - b).abs().max() / b.abs().max())
        assert err < tol, (r, err)


def case_single_layer(device, tol, kind, moe, dtype=torch.float32, n=90, **kw):
    """One layer with one mixer, with and without experts: whole, token by token, and in portions."""
    cfg = O.make_config(mixers=(kind,), moe=moe, **kw)
    sd = slow_decay(O.make_weights(cfg, seed=21))
    toks = tokens(cfg, n, 5)
    want = O.forward(cfg, sd, toks)
    _, eng = build(cfg, sd, device, dtype)
    assert rel_err(feed_in_portions(eng, "w", toks, [n]), want) < tol
    assert rel_err(feed_in_portions(eng, "d", toks, [1]), want) < tol
    assert rel_err(feed_in_portions(eng, "c", toks, [6, 2, 19]), want) < tol


def case_shared_tensors(device, tol, dtype=torch.float32):
    """Layers on another layer's tensors keep a cache and a state of their own: with one pool row for both the second
    would read the first's.  Also a chain of references and one to a later layer."""
    for mixers, shared in (((DELTA, ATT, DELTA, ATT), {2: 0, 3: 1}), ((DELTA, DELTA, DELTA), {1: 0, 2: 1}), ((ATT, ATT), {0: 1})):
        cfg = O.make_config(mixers=mixers, shared=shared)
        sd = slow_decay(O.make_weights(cfg, seed=25))
        toks = tokens(cfg, 50, 8)
        want = O.forward(cfg, sd, toks)
        model, eng = build(cfg, sd, device, dtype)
        for i, j in shared.items():
            assert model.layers[i] is model.layers[j]
        own = [t for t in model.allocate_kv_cache(2, 16) + model.allocate_state(2) if t is not None]
        assert len({b.data_ptr() for _, b in own}) == len(mixers)
        for i, cuts in enumerate(([50], [1], [17, 2, 12])):
            assert rel_err(feed_in_portions(eng, f"s{i}", toks, cuts), want) < tol, (shared, cuts)


def case_prefill_vs_decode(device, tol, dtype=torch.float32, n=58, **cfg_kw):
    cfg = O.make_config(**cfg_kw)
    sd = slow_decay(O.make_weights(cfg, seed=5))
    toks = tokens(cfg, n, 1)
    want = O.forward(cfg, sd, toks)
    _, eng = build(cfg, sd, device, dtype)
    assert rel_err(feed_in_portions(eng, "p", toks, [n]), want) < tol
    assert rel_err(feed_in_portions(eng, "d", toks, [1]), want) < tol           # every token on the decode path
    assert rel_err(feed_in_portions(eng, "pd", toks, [n - 25] + [1] * 25), want) < tol  # windows pass over decoded tokens


def case_portions(device, tol, dtype=torch.float32):
    """Portions cut inside pages (16), the window (11), the convolution's reach (3), the delta rule's blocks (16) and
    chunks (64), down to two tokens."""
    cfg = O.make_config()
    sd = slow_decay(O.make_weights(cfg, seed=7))
    toks = tokens(cfg, 139, 2)
    want = O.forward(cfg, sd, toks)
    _, eng = build(cfg, sd, device, dtype)
    for k, cuts in enumerate(([2], [3, 2, 17, 1, 16, 31], [16], [15, 1, 1, 33], [11, 19], [64, 2], [65, 63, 11], [130, 9],
                              [1, 2], [4, 70], [128, 11])):
        assert rel_err(feed_in_portions(eng, f"c{k}", toks, cuts), want) < tol, cuts


def case_batches(device, tol, dtype=torch.float32, alone=False, long=1):
    """Unequal requests in one batch -- portions beside single tokens, requests that sit out steps and end at
    different times -- give each request the logits it gets alone: the oracle's, or (``alone``) the same engine's
    when it serves the request whole and by itself.  ``long``: the portions' lengths times this."""
    cfg = O.make_config()
    sd = slow_decay(O.make_weights(cfg, seed=9))
    plan = [  # (request, tokens) per step
        [("a", 20 * long), ("b", 2)],
        [("a", 1), ("b", 1), ("c", 17 * long)],
        [("a", 1), ("c", 1), ("d", 16 * long)],
        [("b", 6), ("a", 3), ("d", 1), ("c", 13)],
        [("a", 20 * long), ("d", 1)],
    ]
    lens = {k: sum(n for s in plan for r, n in s if r == k) for k in "abcd"}
    toks = {k: tokens(cfg, n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    _, eng = build(cfg, sd, device, dtype, pool_tokens=sum(-(-n // 16) * 16 for n in lens.values()))
    if alone:
        want = {k: torch.as_tensor(feed_in_portions(eng, k + "0", t, [len(t)]), dtype=torch.float64) for k, t in toks.items()}
    else:
        want = {k: O.forward(cfg, sd, t) for k, t in toks.items()}
    cur = {k: 0 for k in toks}
    got = {k: [] for k in toks}
    for step in plan:
        entries, end = [], []
        for k, n in step:
            entries.append((k, toks[k][cur[k]:cur[k] + n], list(range(n))))
            cur[k] += n
            if cur[k] == lens[k]:
                end.append(k)
        out = eng.feed(entries, end)
        o = 0
        for k, n in step:
            got[k].append(out[o:o + n])
            o += n
    for k in toks:
        assert cur[k] == lens[k]
        assert rel_err(np.concatenate(got[k], 0), want[k]) < tol, k
    assert eng.kv.num_free == eng.kv.num_blocks - 1 and len(eng.sched.free_slots) == 4


def case_reuse(device, tol, dtype=torch.float32):
    """Pages and state slots that were freed are used again: with one slot and a pool of one request's worth, later
    requests land on the earlier ones' pages, convolution inputs and states and still match their oracle."""
    cfg = O.make_config()
    sd = slow_decay(O.make_weights(cfg, seed=11))
    _, eng = build(cfg, sd, device, dtype, slots=1, pool_tokens=64)
    for i, n in enumerate((50, 7, 33, 64, 1)):
        toks = tokens(cfg, n, 20 + i)
        want = O.forward(cfg, sd, toks)
        cuts = [[n], [3, 1], [32, 1], [60, 2, 1, 1], [1]][i]
        assert rel_err(feed_in_portions(eng, f"r{i}", toks, cuts), want) < tol, i
        assert eng.kv.num_free == eng.kv.num_blocks - 1
    # a request that stops mid-way leaves nothing behind either
    eng.feed([("x", tokens(cfg, 40, 30), [])], [])
    eng.feed([], ["x"])
    toks = tokens(cfg, 21, 31)
    assert rel_err(feed_in_portions(eng, "y", toks, [20, 1]), O.forward(cfg, sd, toks)) < tol


def case_long_decode(device, tol, dtype=torch.float32):
    cfg = O.make_config(window=33)
    sd = slow_decay(O.make_weights(cfg, seed=13))
    toks = tokens(cfg, 150, 3)
    want = O.forward(cfg, sd, toks)
    _, eng = build(cfg, sd, device, dtype)
    assert rel_err(feed_in_portions(eng, "l", toks, [6] + [1] * 144), want) < tol


VARIANTS = [
    # one kv head everywhere, whole-head rotary, value sizes above the key sizes, a window of one position (only itself),
    # one tap; one expert in one group
    dict(width=40, vocab=33, heads=3, kv_heads=1, dim=10, vdim=24, rot_dims=10, rot_base=7.0, scale=1.0, window=1, dheads=4,
         dkv_heads=1, ddim=6, dvdim=33, conv=1, experts=1, groups=(1, 1), top=1, ff=8, route_scale=1.0, embed_scale=1.0),
    # heads == kv heads, no rotary, a window longer than the prompt; key sizes above the value sizes, two taps; every expert
    # chosen, a group per expert
    dict(heads=2, kv_heads=2, dim=72, vdim=72, rot_dims=0, scale=0.1, window=500, dheads=2, dkv_heads=2, ddim=72, dvdim=5,
         conv=2, experts=4, groups=(4, 4), top=4, ff=16),
    # one head each, sizes of 1; a group open out of many, no shared expert
    dict(width=56, heads=1, kv_heads=1, dim=2, vdim=1, rot_dims=2, window=2, dheads=1, dkv_heads=1, ddim=1, dvdim=1, conv=3,
         experts=10, groups=(5, 1), top=2, shared_ff=0),
    # a width and a vocabulary that are multiples of nothing useful (rows of 60 bytes), odd head sizes, six taps
    dict(width=30, vocab=77, heads=6, kv_heads=3, dim=6, vdim=10, rot_dims=2, window=6, dheads=9, dkv_heads=3, ddim=7,
         dvdim=11, conv=6, experts=6, groups=(2, 1), top=3, ff=9, shared_ff=11, eps=0.1),
    # head sizes past 64 and past 128
    dict(mixers=(DELTA,), dheads=2, dkv_heads=1, ddim=100, dvdim=132, conv=4, width=64, moe=False),
    dict(mixers=(DELTA, ATT), dheads=2, dkv_heads=2, ddim=200, dvdim=40, heads=2, kv_heads=1, dim=136, vdim=16, width=64,
         moe=False),
    # a layer without a feed-forward among layers with one
    dict(mixers=(ATT, DELTA, ATT), moe=(True, False, False), groups=(1, 1), top=3, window=20),
]


def case_other_sizes(device, tol, dtype=torch.float32):
    """Sizes where things the usual configs make equal differ, or are 1."""
    for i, kw in enumerate(VARIANTS):
        cfg = O.make_config(**kw)
        sd = O.make_weights(cfg, seed=40 + i)
        toks = tokens(cfg, 29, 40 + i)
        want = O.forward(cfg, sd, toks)
        _, eng = build(cfg, sd, device, dtype)
        assert rel_err(feed_in_portions(eng, "w", toks, [29]), want) < tol, i
        assert rel_err(feed_in_portions(eng, "c", toks, [5, 1, 2]), want) < tol, i


def case_mixed_layers(device, tol, dtype=torch.float32):
    """Layers of one model with different head counts, windows, rotations, state sizes, taps and experts."""
    a = O.make_config()
    b = O.make_config(heads=2, kv_heads=1, dim=12, vdim=20, window=5, rot_dims=4, rot_base=9.0, scale=0.8, dheads=2,
                      dkv_heads=2, ddim=20, dvdim=9, conv=2, experts=4, groups=(2, 1), top=2, route_scale=0.5, ff=12,
                      shared_ff=0)
    c = O.make_config(window=23, rot_dims=0, dheads=4, dkv_heads=1, ddim=33, dvdim=36, conv=5, experts=8, groups=(1, 1), top=5)
    cfg = dict(a, layers=b["layers"] + a["layers"] + c["layers"] + [dict(b["layers"][0], weights_of=0)])
    sd = O.make_weights(cfg, seed=27)
    toks = tokens(cfg, 44, 9)
    want = O.forward(cfg, sd, toks)
    _, eng = build(cfg, sd, device, dtype)
    for i, cuts in enumerate(([44], [1], [13, 2, 8])):
        assert rel_err(feed_in_portions(eng, f"m{i}", toks, cuts), want) < tol, cuts


def case_first_tokens(device, tol, dtype=torch.float32):
    """Position 0 alone (one key, a state and a convolution that start from zeros in a used slot), then 1, 2."""
    cfg = O.make_config()
    sd = slow_decay(O.make_weights(cfg, seed=17))
    _, eng = build(cfg, sd, device, dtype, slots=1)
    eng.feed([("warm", tokens(cfg, 30, 50), [])], ["warm"])  # leave a state and pages behind
    for n in (1, 2, 3, 5):
        toks = tokens(cfg, n, 60 + n)
        want = O.forward(cfg, sd, toks)
        assert rel_err(feed_in_portions(eng, f"f{n}", toks, [1]), want) < tol
        assert rel_err(feed_in_portions(eng, f"g{n}", toks, [n]), want) < tol


def case_sharp_far_keys(device, tol, dtype=torch.float32):
    """A softmax scale large enough that every query picks out single keys, many of them far back and across page
    borders: a key read from the wrong place changes the logits outright.  300 tokens, a window of 110, the last 40
    decoded one by one, portions cut off the page grid."""
    cfg = O.make_config(mixers=(ATT, ATT), moe=False, scale=5.0, window=110, kv_heads=1)
    sd = O.make_weights(cfg, seed=29)
    toks = tokens(cfg, 300, 6)
    want = O.forward(cfg, sd, toks)
    _, eng = build(cfg, sd, device, dtype)
    assert rel_err(feed_in_portions(eng, "s", toks, [300]), want) < tol
    assert rel_err(feed_in_portions(eng, "t", toks, [97, 130, 33] + [1] * 40), want) < tol


def case_window_edges(device, tol, dtype=torch.float32, bs=16, ctx=75, d=80, windows=None):
    """The attention op alone on crafted keys: key j is 30 e_j, so a query e_p scores 30 on position p and 0 elsewhere,
    and the softmax weight of an asked-for visible key is ~1.  Head 0 asks for the oldest key of the query's window,
    head 1 for the key before it, head 2 for the query's own position.  A hidden key's asker must see the flat average
    of the visible keys' values instead.  In a prompt's portion that follows cached context and for a decoded token;
    windows that end on, before and after page and tile borders; pages out of order."""
    from githubrepostorag_amd.ops.attention import AttnMetadata, sink_attention

    dev = torch.device(device)
    H, G, vd = 3, 1, 16
    nb = -(-ctx // bs)
    for window in windows or (1, 2, 5, bs, bs + 1, 40, 63, 64, 65, 75, 200):
        g = torch.Generator().manual_seed(window)
        perm = (torch.randperm(nb, generator=g) + 1).to(torch.int32)
        kc = torch.zeros(nb + 1, G, bs, d, dtype=dtype, device=dev)
        vc = torch.zeros(nb + 1, G, bs, vd, dtype=dtype, device=dev)
        for j in range(ctx):
            kc[perm[j // bs], 0, j % bs, j] = 30.0
            vc[perm[j // bs], 0, j % bs, 0] = j + 1.0  # the value names its position
        for qlen in (33, 9, 1):  # (33 queries in bf16: the matrix-core kernel)
            q = torch.zeros(qlen, H, d)
            asked = []
            for n, p in enumerate(range(ctx - qlen, ctx)):
                lo = max(0, p - window + 1)
                asked.append((p, (lo, lo - 1, p)))
                for hh, j in enumerate(asked[-1][1]):
                    if j >= 0:
                        q[n, hh, j] = 1.0
            i32 = dict(dtype=torch.int32, device=dev)
            meta = AttnMetadata(q_start=torch.tensor([0, qlen], **i32), ctx_len=torch.tensor([ctx], **i32),
                                block_tables=perm.view(1, nb).to(dev), slot_mapping=torch.zeros(qlen, **i32),
                                max_q_len=qlen, num_seqs=1, num_tokens=qlen, is_decode=qlen == 1)
            got = sink_attention(q.to(dtype).to(dev), kc, vc, meta, 1.0, None, window=window).float().cpu().view(qlen, H, vd)
            for n, (p, row) in enumerate(asked):
                seen = O.visible(p, window)
                flat = sum(j + 1.0 for j in seen) / len(seen)
                for hh, j in enumerate(row):
                    want = j + 1.0 if j in seen else flat
                    assert abs(float(got[n, hh, 0]) - want) < tol * ctx, (window, qlen, p, hh)


def case_generate(device, dtype=torch.float32, graphs=False, mixed=False, window=1, max_batched=4096, tol=2e-3,
                  **cfg_kw):
    """Greedy generation through LLMEngine.generate (scheduler, chunked prefill, sampler, decode steps): every
    generated token is the oracle's arg-max given the tokens before it (up to a near-tie)."""
    from githubrepostorag_amd.engine.sequence import SamplingParams

    cfg = O.make_config(**cfg_kw)
    sd = slow_decay(O.make_weights(cfg, seed=19))
    _, eng = build(cfg, sd, device, dtype, slots=3, pool_tokens=256, graphs=graphs, mixed=mixed, window=window,
                   max_batched=max_batched)
    prompts = [tokens(cfg, n, 70 + i) for i, n in enumerate((5, 23, 11, 2))]  # 4 prompts on 3 slots: one waits
    outs = eng.generate(prompts, SamplingParams(max_tokens=14, temperature=0.0, ignore_eos=True))
    for p, c in zip(prompts, outs):
        assert len(c.token_ids) == 14
        logits = O.forward(cfg, sd, p + c.token_ids[:-1])
        for j, t in enumerate(c.token_ids):
            row = logits[len(p) - 1 + j]
            assert float(row.max() - row[t]) < tol * float(row.std()), (len(p), j)
    assert eng.kv.num_free == eng.kv.num_blocks - 1
