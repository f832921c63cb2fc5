"""A plain float64 implementation of the Vudivik decoder, one function per mechanism, written from the design's
equations with loops over tokens.  Slow on purpose; it shares no code with the engine.

Weights: a dict name -> tensor (any dtype; floats are used as float64).  Config: the config.json dict.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


def relu2(z):
    return torch.clamp(z, min=0.0) ** 2


def frequencies(rot):
    """The turn per position of every pair: base^(-2i / dims), wavelengths above original / low stretched by factor,
    those below original / high kept, a linear blend (in original / wavelength) between the two."""
    out = []
    sc = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_halves(x, pos, freqs):
    """Entries i and i + dims/2 of the first dims = 2 len(freqs) of the last axis form pair i, turned by
    pos * freqs[i]."""
    out = x.clone()
    half = len(freqs)
    for i, f in enumerate(freqs):
        c, s = math.cos(pos * f), math.sin(pos * f)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def visible(i, window, keep):
    """The positions query i sees: itself and the window - 1 before it, and the first ``keep`` of the sequence."""
    return [j for j in range(i + 1) if i - j < window or j < keep]


def attention(h, W, m, eps):
    """Grouped-query attention with biased projections, an RMS norm per q / k head, scaled rotary, a sliding window that
    keeps the first tokens, plain softmax.  h [T, width] -> [T, width]."""
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    rot = m.get("rot")
    fr = frequencies(rot) if rot else []
    mask = m.get("mask") or {}
    win, keep = mask.get("size") or T, mask.get("keep_first", 0)
    q = rms_unit((h @ W("q").T + W("q.b")).view(T, H, d), eps) * W("q.norm")
    k = rms_unit((h @ W("k").T + W("k.b")).view(T, G, d), eps) * W("k.norm")
    v = (h @ W("v").T + W("v.b")).view(T, G, vd)
    kr = torch.stack([rotate_halves(k[t], t, fr) for t in range(T)]).repeat_interleave(H // G, dim=1)
    vr = v.repeat_interleave(H // G, dim=1)  # query head h reads key / value head h // (H / G)
    out = torch.zeros(T, H, vd, dtype=F64)
    for i in range(T):
        seen = torch.tensor(visible(i, win, keep))
        qi = rotate_halves(q[i], i, fr)
        p = torch.softmax((kr[seen] * qi).sum(-1) * m["scale"], 0)
        out[i] = (p[:, :, None] * vr[seen]).sum(0)
    return out.reshape(T, H * vd) @ W("o").T


def short_conv(x, w, b):
    """Per channel: b + sum_j w[:, j] x[t - (taps - 1) + j], nothing before the start; then silu."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        acc = b.clone()
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                acc = acc + w[:, j] * x[s]
        out[t] = silu(acc)
    return out


def selective_scan(x, dt, A, B, C, D):
    """Per channel and state number: S <- exp(dt A) S + dt x B, y = sum S C + D x.  x, dt [T, inner]; A [inner, N];
    B, C [T, N]."""
    S = torch.zeros_like(A)
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h, W, m):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    p = h @ W("in").T
    x = short_conv(p[:, :inner], W("conv"), W("conv.b"))
    z = p[:, inner:]
    low = x @ W("x").T
    dt = softplus(low[:, :R] @ W("dt").T + W("dt.b"))
    y = selective_scan(x, dt, -torch.exp(W("A_log")), low[:, R:R + N], low[:, R + N:], W("D"))
    return (y * silu(z)) @ W("o").T


def parallel(h, W, m, eps):
    """Half the sum of the two mixers' outputs, each RMS-normed first."""
    left = rms_unit(attention(h, lambda n: W("left." + n), m["left"], eps), eps) * W("left.out")
    right = rms_unit(mamba(h, lambda n: W("right." + n), m["right"]), eps) * W("right.out")
    return 0.5 * (left + right)


def dense(h, W, prefix=""):
    return relu2(h @ W(prefix + "up").T) @ W(prefix + "down").T


def route(h, W, r):
    """Per token [(expert, weight)]: the softmax scores choose with the correction added, weigh without it."""
    s = torch.softmax(h @ W("router").T, -1)
    c = s + W("correction")
    out = []
    for t in range(h.shape[0]):
        chosen = sorted(range(s.shape[1]), key=lambda e: (-float(c[t, e]), e))[: r["top"]]
        out.append([(e, s[t, e]) for e in chosen])
    return out


def moe(h, W, f):
    """Routed experts; the numbers from ``experts`` up are identity experts, which return their input."""
    r = f["router"]
    out = torch.zeros_like(h)
    for t, choice in enumerate(route(h, W, r)):
        for e, w in choice:
            out[t] += w * (dense(h[t:t + 1], W, f"e{e}.")[0] if e < r["experts"] else h[t])
    return out


def tensors_of(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def logits_and_taps(cfg, sd, toks):
    """-> (logits [T, vocab], residual after every layer [layers, T, width]), float64."""
    sd = {k: v.to(F64) for k, v in sd.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = sd["embed"][torch.tensor(toks)]
    taps = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{tensors_of(cfg, i)}."
        y = parallel(x, lambda n: sd[p + "mix." + n], L["mixer"], eps)
        x = x + mult * rms_unit(y, eps) * sd[p + "norm1"]
        f = L.get("mlp")
        if f is not None:
            W = lambda n: sd[p + "mlp." + n]
            y = moe(x, W, f) if f["kind"] == "moe" else dense(x, W)
            x = x + mult * rms_unit(y, eps) * sd[p + "norm2"]
        taps.append(x.clone())
    return (rms_unit(x, eps) * sd["final.norm"]) @ sd["head"].T, torch.stack(taps)


def forward(cfg, sd, toks):
    return logits_and_taps(cfg, sd, toks)[0]


# ------------------------------------------------------------------------------------------------ test models
DENSE, MOE = "dense", "moe"


def make_config(mlps=(DENSE, MOE, None), shared=None, vocab=96, width=48, heads=4, kv_heads=2, dim=16, vdim=8, window=11,
                keep=3, rot_dims=8, rot_base=100.0, scaling=(4.0, 1.0, 4.0, 40), scale=0.4, inner=36, state=6, dt_rank=5,
                taps=4, ff=40, experts=5, identity=2, top=3, expert_ff=20, mult=0.6, eps=1e-5):
    """``mlps``: the feed-forward of every layer; ``shared`` {i: j}: layer i runs on layer j's tensors."""
    layers = []
    for i, kind in enumerate(mlps):
        left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                "mask": {"size": window, "keep_first": keep}, "rot": {"dims": rot_dims, "base": rot_base}}
        if scaling is not None:
            left["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
        right = {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": taps}
        mlp = None
        if kind == DENSE:
            mlp = {"kind": "dense", "ff": ff}
        elif kind == MOE:
            mlp = {"kind": "moe", "expert": {"ff": expert_ff},
                   "router": {"experts": experts, "identity": identity, "top": top}}
        e = {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}
        if shared and i in shared:
            e["weights_of"] = shared[i]
        layers.append(e)
    return {"architecture": "Vudivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "layers": layers}


def make_weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(4321 + seed)
    W = cfg["width"]

    def r(*shape, s=None):
        s = 1.0 / math.sqrt(shape[-1]) if s is None else s
        return (torch.randn(*shape, generator=g) * s).to(dtype)

    def around(v, n, s=0.15):
        return (v + s * torch.randn(n, generator=g)).to(dtype)

    sd = {"embed": r(cfg["vocab"], W, s=1.0), "head": r(cfg["vocab"], W), "final.norm": around(1.0, W)}
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, a, s = f"l{i}.", L["mixer"]["left"], L["mixer"]["right"]
        H, d, vd = a["heads"], a["dim"], a["vdim"]
        G = a.get("kv_heads", H)
        m = p + "mix.left."
        sd.update({m + "q": r(H * d, W), m + "q.b": r(H * d, s=0.5), m + "k": r(G * d, W), m + "k.b": r(G * d, s=0.5),
                   m + "v": r(G * vd, W), m + "v.b": r(G * vd, s=0.5), m + "q.norm": around(1.0, d, 0.3),
                   m + "k.norm": around(1.0, d, 0.3), m + "o": r(W, H * vd), m + "out": around(1.0, W)})
        inner, N, R, K = s["inner"], s["state"], s["dt_rank"], s["conv"]
        m = p + "mix.right."
        sd.update({m + "in": r(2 * inner, W), m + "conv": r(inner, K, s=0.6), m + "conv.b": r(inner, s=0.2),
                   m + "x": r(R + 2 * N, inner), m + "dt": r(inner, R), m + "dt.b": r(inner, s=1.0),
                   m + "A_log": (torch.rand(inner, N, generator=g) * 3.5 - 2.5).to(dtype), m + "D": around(1.0, inner, 0.3),
                   m + "o": r(W, inner), m + "out": around(1.0, W)})
        sd[p + "norm1"] = around(1.0, W)
        f = L.get("mlp")
        if f is None:
            continue
        sd[p + "norm2"] = around(1.0, W)
        if f["kind"] == "dense":
            sd.update({p + "mlp.up": r(f["ff"], W), p + "mlp.down": r(W, f["ff"])})
            continue
        F, rt = f["expert"]["ff"], f["router"]
        for e in range(rt["experts"]):
            sd.update({p + f"mlp.e{e}.up": r(F, W), p + f"mlp.e{e}.down": r(W, F)})
        E = rt["experts"] + rt.get("identity", 0)
        sd[p + "mlp.router"] = r(E, W, s=1.5 / math.sqrt(W))
        sd[p + "mlp.correction"] = r(E, s=0.15)
    return sd
