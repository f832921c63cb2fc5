"""A plain float64 implementation of the Kapanex decoder, one function per mechanism, written from the design's
equations with loops over tokens.  Slow on purpose; it shares no code with the engine.

Weights: a dict name -> tensor (any dtype; floats are used as float64).  Config: the config.json dict.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def layer_norm(x, w, eps):
    """(x - mean) / sqrt(mean squared deviation + eps) * w over the last axis, no bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


def short_conv(x, w):
    """Per channel: sum_j w[:, j] x[t - (taps - 1) + j], nothing before the start; then silu."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return silu(out)


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d]; v [T, H, vd]; g, beta [T, H].  Per head S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.
    -> o [T, H, vd], the last state [H, d, vd]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out, S


def delta(h, W, m, eps):
    """The gated delta-rule mixer.  h [T, width] -> [T, width]."""
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    q = short_conv(h @ W("q").T, W("q.conv")).view(T, G, d)
    k = short_conv(h @ W("k").T, W("k.conv")).view(T, G, d)
    v = short_conv(h @ W("v").T, W("v.conv")).view(T, H, vd)
    q = (unit(q) * d ** -0.5).repeat_interleave(H // G, dim=1)
    k = unit(k).repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(h @ W("b").T)
    g = torch.exp(-torch.exp(W("A_log")) * softplus(h @ W("a").T + W("dt_bias")))
    o, _ = delta_rule(q, k, v, g, beta)
    o = rms_unit(o, eps) * W("norm") * silu((h @ W("g").T).view(T, H, vd))
    return o.reshape(T, H * vd) @ W("o").T


def rotate_halves(x, pos, dims, base):
    """Entries i and i + dims/2 of the first ``dims`` of the last axis form pair i, turned by pos * base^(-2i/dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = pos * float(base) ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = x[..., i], x[..., i + dims // 2]
        out[..., i] = u * c - v * s
        out[..., i + dims // 2] = v * c + u * s
    return out


def visible(i, window):
    """The positions query i sees: itself and the window - 1 before it."""
    return [j for j in range(i + 1) if i - j < window]


def attention(h, W, m, eps):
    """Grouped-query attention in a sliding window; q and k are rotated, then divided by their root mean square."""
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    win = (m.get("mask") or {}).get("size") or T
    q, k, v = (h @ W("q").T).view(T, H, d), (h @ W("k").T).view(T, G, d), (h @ W("v").T).view(T, G, vd)
    turn = lambda x: torch.stack([rms_unit(rotate_halves(x[t], t, rot["dims"], rot["base"]), eps) for t in range(T)])
    q, k = turn(q), turn(k).repeat_interleave(H // G, dim=1)  # query head h reads key / value head h // (H / G)
    v = v.repeat_interleave(H // G, dim=1)
    out = torch.zeros(T, H, vd, dtype=F64)
    for i in range(T):
        seen = torch.tensor(visible(i, win))
        p = torch.softmax((k[seen] * q[i]).sum(-1) * m["scale"], 0)
        out[i] = (p[:, :, None] * v[seen]).sum(0)
    return out.reshape(T, H * vd) @ W("o").T


def glu(h, W, prefix):
    return (silu(h @ W(prefix + "gate").T) * (h @ W(prefix + "up").T)) @ W(prefix + "down").T


def route(h, W, r):
    """Per token [(expert, weight)]: sigmoid scores; a group counts as much as its two best experts together; the best
    ``top`` experts of the ``keep`` best groups, their scores made to sum to 1 and multiplied by ``scale``."""
    s = torch.sigmoid(h @ W("router").T)
    E = s.shape[1]
    gr = r.get("groups") or {"count": 1, "keep": 1}
    per = E // gr["count"]
    out = []
    for t in range(h.shape[0]):
        worth = [float(sum(sorted((s[t, e] for e in range(n * per, (n + 1) * per)), reverse=True)[:2]))
                 for n in range(gr["count"])]
        best = sorted(range(gr["count"]), key=lambda n: (-worth[n], n))[: gr["keep"]]
        open_ = [e for e in range(E) if e // per in best]
        chosen = sorted(open_, key=lambda e: (-float(s[t, e]), e))[: r["top"]]
        total = sum(s[t, e] for e in chosen) + 1e-20
        out.append([(e, s[t, e] / total * r["scale"]) for e in chosen])
    return out


def moe(h, W, f):
    """The routed experts' weighted sum and the shared expert under its gate."""
    out = torch.zeros_like(h)
    for t, choice in enumerate(route(h, W, f["router"])):
        for e, w in choice:
            out[t] += w * glu(h[t:t + 1], W, f"e{e}.")[0]
    if f.get("shared"):
        out = out + torch.sigmoid(h @ W("shared.sg").T) * glu(h, W, "shared.")
    return out


def tensors_of(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def logits_and_taps(cfg, sd, toks):
    """-> (logits [T, vocab], residual after every layer [layers, T, width]), float64."""
    sd = {k: v.to(F64) for k, v in sd.items()}
    eps = cfg["norm"]["eps"]
    x = sd["embed"][torch.tensor(toks)] * cfg["embedding"]["scale"]
    taps = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{tensors_of(cfg, i)}."
        mixer = {"delta": delta, "attention": attention}[L["type"]]
        y = mixer(layer_norm(x, sd[p + "norm1"], eps), lambda n: sd[p + "mix." + n], L["mixer"], eps)
        if L.get("mlp") is not None:
            y = y + moe(layer_norm(x, sd[p + "norm2"], eps), lambda n: sd[p + "mlp." + n], L["mlp"])
        x = x + y
        taps.append(x.clone())
    return layer_norm(x, sd["final.norm"], eps) @ sd["head"].T, torch.stack(taps)


def forward(cfg, sd, toks):
    return logits_and_taps(cfg, sd, toks)[0]


# ------------------------------------------------------------------------------------------------ test models
DELTA, ATT = "delta", "attention"


def make_config(mixers=(DELTA, ATT, DELTA), shared=None, moe=True, vocab=96, width=48, heads=4, kv_heads=2, dim=16, vdim=8,
                window=11, rot_dims=8, rot_base=100.0, scale=1.5, dheads=6, dkv_heads=3, ddim=12, dvdim=20, conv=4,
                experts=6, top=2, groups=(3, 2), route_scale=1.7, ff=20, shared_ff=28, embed_scale=3.0, eps=1e-5):
    """``mixers``: the mixer of every layer; ``shared`` {i: j}: layer i runs on layer j's tensors; ``moe``: whether the
    layers have a feed-forward, one answer or one per layer."""
    layers = []
    for i, kind in enumerate(mixers):
        if kind == DELTA:
            m = {"heads": dheads, "kv_heads": dkv_heads, "dim": ddim, "vdim": dvdim, "conv": conv}
        else:
            m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                 "mask": {"size": window}, "rot": {"dims": rot_dims, "base": rot_base}}
        mlp = {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared_ff} if shared_ff else None,
               "router": {"experts": experts, "top": top, "scale": route_scale,
                          "groups": {"count": groups[0], "keep": groups[1]}}}
        e = {"type": kind, "mixer": m, "mlp": mlp if (moe if isinstance(moe, bool) else moe[i]) else None}
        if shared and i in shared:
            e["weights_of"] = shared[i]
        layers.append(e)
    return {"architecture": "Kapanex", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "layers": layers}


def make_weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(8765 + seed)
    W = cfg["width"]

    def r(*shape, s=None):
        s = 1.0 / math.sqrt(shape[-1]) if s is None else s
        return (torch.randn(*shape, generator=g) * s).to(dtype)

    def around(v, n, s=0.15):
        return (v + s * torch.randn(n, generator=g)).to(dtype)

    sd = {"embed": r(cfg["vocab"], W, s=1.0 / cfg["embedding"]["scale"]), "head": r(cfg["vocab"], W),
          "final.norm": around(1.0, W)}
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m, a = f"l{i}.", f"l{i}.mix.", L["mixer"]
        H, d, vd = a["heads"], a["dim"], a["vdim"]
        G = a.get("kv_heads", H)
        sd[p + "norm1"] = around(1.0, W)
        if L["type"] == DELTA:
            sd.update({m + "q": r(G * d, W), m + "k": r(G * d, W), m + "v": r(H * vd, W), m + "b": r(H, W), m + "a": r(H, W),
                       m + "g": r(H * vd, W), m + "A_log": (torch.rand(H, generator=g) * 2.0 - 1.5).to(dtype),
                       m + "dt_bias": around(-1.5, H, 1.0), m + "norm": around(1.0, vd, 0.3)})
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * vd)):
                sd[m + n + ".conv"] = r(rows, a["conv"], s=0.6)
        else:
            sd.update({m + "q": r(H * d, W), m + "k": r(G * d, W), m + "v": r(G * vd, W)})
        sd[m + "o"] = r(W, H * vd)
        f = L.get("mlp")
        if f is None:
            continue
        sd[p + "norm2"] = around(1.0, W)
        parts = [(f"mlp.e{e}.", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
        if f.get("shared"):
            parts.append(("mlp.shared.", f["shared"]["ff"]))
            sd[p + "mlp.shared.sg"] = r(1, W)
        for n, F in parts:
            sd.update({p + n + "gate": r(F, W), p + n + "up": r(F, W), p + n + "down": r(W, F)})
        sd[p + "mlp.router"] = r(f["router"]["experts"], W, s=1.5 / math.sqrt(W))
    return sd
