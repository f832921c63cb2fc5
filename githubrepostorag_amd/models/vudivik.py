"""Vudivik: a decoder that norms what its sublayers give rather than what they read, with windowed attention beside a
selective scan in every layer, on the paged-KV engine.

The layer list is data (models/configs.py HybridConfig, arch "vudivik").  With the fp32 residual x, the residual
multiplier m and the RMS norm unit(v) = v / sqrt(mean(v^2) + eps),

    x <- x + m * unit(mixer(x)) * w_norm1;   x <- x + m * unit(ff(x)) * w_norm2
    mixer(x) = (unit(left(x)) * w_left + unit(right(x)) * w_right) / 2

The sublayers read x itself (its bf16 rounding in the bf16 mode; the router reads the fp32 residual).  A layer may run
on another layer's tensors; its K/V cache and its recurrent state are its own.

Left: grouped-query softmax attention over the last ``window`` positions and the first ``keep_first`` of the sequence;
  biased projections, an RMS norm per query / key head, rotary on halves of the first rot dims with stretched long
  wavelengths                                   [grag_rope_vnorm_store with bias / qw / kw, grag_sink_attn_* with keep]
Right: causal convolution + SiLU, then a selective scan whose decay differs per channel and state number, gated by
  SiLU(z); the convolution's last inputs and the fp32 state are carried per sequence
                                                                                  [grag_causal_conv, grag_chan_scan]
Feed-forward: W_down max(W_up x, 0)^2, dense [grag_relu2] or a mixture of experts: softmax scores over the experts and
  some identity experts, chosen by score + correction, weighted by the score alone
                                                                     [grag_moe_route, grag_moe_align, grag_moe_gemm]

Per layer all input projections of both mixers are one GEMM (q | k | v | conv input | z), and every sublayer boundary is
one kernel: the branches' norms, their sum, the norm of the sum, x += m * that, the next sublayer's input
[grag_postnorm_residual].  Activations are bf16 (or fp32 end to end with dtype=torch.float32: the GEMMs then run in true
fp32); the residual, norms, positions, angles, scores, softmax weights, router, step sizes, decays and states are fp32
in both.
"""
from __future__ import annotations

import math

import torch

from ..ops.attention import AttnMetadata, sink_attention
from ..ops.elementwise import relu2_, rope_table, rope_vnorm_store
from ..ops.linear import linear
from ..ops.moe import moe_experts, moe_route
from ..ops.norm import embed_gather_f32, postnorm_residual
from ..ops.recurrent import causal_conv, pad_step_matrix, selective_scan
from ..parallel.comm import Group
from .configs import HybridConfig, MLPSpec


class _Layer:
    __slots__ = ("spec", "norm1", "norm2", "wp", "bias", "off", "qnorm", "knorm", "rope", "wol", "lout", "convw", "convb",
                 "wx", "wdt", "dtb", "A", "skip", "wor", "rout", "wup", "wdown", "wr", "corr")


def _pad8(t: torch.Tensor) -> torch.Tensor:
    """Rows padded with zeros to a multiple of 8 (projection matrices: 16-byte output rows)."""
    pad = -t.shape[0] % 8
    return t if not pad else torch.cat([t, torch.zeros(pad, *t.shape[1:], dtype=t.dtype)], 0)


def init_state_dict(cfg: HybridConfig, seed: int = 0, std: float | None = None) -> dict:
    """Random weights under the checkpoint's tensor names (bf16; benches and tests -- not a trained model)."""
    g = torch.Generator().manual_seed(seed * 1000003 + 17)
    W = cfg.hidden_size

    def r(*shape, s=None):
        s = (1.0 / math.sqrt(shape[-1])) if s is None else s
        return (torch.randn(*shape, generator=g) * (std or s)).to(torch.bfloat16)

    def around(v, n, s=0.1):
        return (v + s * torch.randn(n, generator=g)).to(torch.bfloat16)

    sd = {"embed": r(cfg.vocab_size, W, s=1.0), "head": r(cfg.vocab_size, W), "final.norm": around(1.0, W)}
    for i, L in enumerate(cfg.layers):
        if L.weights_of is not None:
            continue
        p, a, c, f = f"l{i}.", L.mixer.left, L.mixer.right, L.mlp
        m = p + "mix.left."
        for n, rows in (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim)):
            sd[m + n], sd[m + n + ".b"] = r(rows, W), r(rows, s=0.2)
        sd.update({m + "q.norm": around(1.0, a.dim), m + "k.norm": around(1.0, a.dim), m + "o": r(W, a.heads * a.vdim),
                   m + "out": around(1.0, W)})
        m = p + "mix.right."
        sd.update({m + "in": r(2 * c.inner, W), m + "conv": r(c.inner, c.taps, s=0.5), m + "conv.b": r(c.inner, s=0.2),
                   m + "x": r(c.dt_rank + 2 * c.state, c.inner), m + "dt": r(c.inner, c.dt_rank),
                   m + "dt.b": around(-3.0, c.inner, 1.0),
                   m + "A_log": torch.log(1.0 + torch.rand(c.inner, c.state, generator=g) * c.state).to(torch.bfloat16),
                   m + "D": around(1.0, c.inner, 0.3), m + "o": r(W, c.inner), m + "out": around(1.0, W)})
        sd[p + "norm1"] = around(1.0, W)
        if f is None:
            continue
        sd[p + "norm2"] = around(1.0, W)
        if isinstance(f, MLPSpec):
            sd[p + "mlp.up"], sd[p + "mlp.down"] = r(f.ff, W), r(W, f.ff)
            continue
        for e in range(f.experts):
            sd[p + f"mlp.e{e}.up"], sd[p + f"mlp.e{e}.down"] = r(f.ff, W), r(W, f.ff)
        sd[p + "mlp.router"] = r(f.experts + f.identity, W, s=1.0 / math.sqrt(W))
        sd[p + "mlp.correction"] = r(f.experts + f.identity, s=0.02)
    return sd


class VudivikModel:
    has_state = True  # recurrent state per sequence slot: the engine allocates it and never reuses cached prefixes

    def __init__(self, cfg: HybridConfig, device="cuda", dtype=torch.bfloat16, tp: Group | None = None,
                 seed: int = 0, state_dict: dict | None = None, init_std: float | None = None):
        assert cfg.arch == "vudivik", cfg.arch
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp = tp or Group([0])
        if not self.tp.trivial:
            raise NotImplementedError("the Vudivik decoder runs on one GPU per replica (no tensor parallelism)")
        if cfg.loop_stop > cfg.loop_start:
            raise ValueError("the Vudivik design has no looped layers")
        # the engine sizes the decode attention's split-KV scratch (hq * head_dim floats per row and split) and
        # picks its split plan (hkv) from these: the widest attention among the layers
        att = [L.mixer.left for L in cfg.layers]
        self.hq = max([a.heads for a in att], default=1)
        self.hkv = min([a.kv_heads for a in att], default=1)
        self.head_dim = max([a.vdim for a in att], default=1)
        self.runs = cfg.layer_runs()
        self._tables: dict = {}
        self._max_pos = 0
        self._load(state_dict if state_dict is not None else init_state_dict(cfg, seed, init_std))
        self.prepare(4096)

    # ------------------------------------------------------------------ weights
    def _load(self, sd: dict):
        cfg, dev, dt = self.cfg, self.device, self.dtype
        W = cfg.hidden_size

        def expect(name, *shape):
            if name not in sd:
                raise KeyError(f"the checkpoint has no tensor {name!r}")
            if tuple(sd[name].shape) != shape:
                raise ValueError(f"{name}: expected {list(shape)}, found {list(sd[name].shape)}")
            return sd[name]

        def act(t):  # a GEMM operand: the activation dtype
            return t.to(device=dev, dtype=dt).contiguous()

        def f32(name, *shape):
            return expect(name, *shape).to(device=dev, dtype=torch.float32).contiguous()

        self.embed = act(expect("embed", cfg.vocab_size, W))
        # LM head rows padded to a multiple of 8: the sampler reads logit rows 8 at a time (zero rows, cut off
        # again in compute_logits)
        self.head = act(_pad8(expect("head", cfg.vocab_size, W)))
        self.final_norm = f32("final.norm", W)
        own = {}
        for i, spec in enumerate(cfg.layers):
            if spec.weights_of is not None:
                continue
            L = own[i] = _Layer()
            for n in _Layer.__slots__:
                setattr(L, n, None)
            L.spec = spec
            a, c, f = spec.mixer.left, spec.mixer.right, spec.mlp
            p, m, r = f"l{i}.", f"l{i}.mix.left.", f"l{i}.mix.right."
            q, k, v = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim
            # one input projection for both mixers; the attention's columns padded to 8 so that the conv input and z
            # start on 16-byte boundaries.  The biases are added in fp32 by the kernel that norms and rotates.
            L.wp = act(_pad8(torch.cat([_pad8(torch.cat([expect(m + "q", q, W), expect(m + "k", k, W),
                                                         expect(m + "v", v, W)], 0)),
                                        expect(r + "in", 2 * c.inner, W)], 0)))
            base = -(-(q + k + v) // 8) * 8
            L.off = (0, q, q + k, base, base + c.inner)  # q | k | v | conv input | z
            L.bias = torch.cat([expect(m + "q.b", q), expect(m + "k.b", k), expect(m + "v.b", v)]).to(
                device=dev, dtype=torch.float32).contiguous()
            L.qnorm, L.knorm = f32(m + "q.norm", a.dim), f32(m + "k.norm", a.dim)
            L.rope = (a.rot_dims, a.rot_base, a.scaling) if a.rot_dims else None
            L.wol, L.lout = act(expect(m + "o", W, a.heads * a.vdim)), f32(m + "out", W)
            L.convw, L.convb = f32(r + "conv", c.inner, c.taps), f32(r + "conv.b", c.inner)
            L.wx = act(_pad8(expect(r + "x", c.dt_rank + 2 * c.state, c.inner)))
            L.wdt = act(pad_step_matrix(expect(r + "dt", c.inner, c.dt_rank)))
            L.dtb, L.skip = f32(r + "dt.b", c.inner), f32(r + "D", c.inner)
            L.A = (-torch.exp(expect(r + "A_log", c.inner, c.state).double())).to(device=dev, dtype=torch.float32).contiguous()
            L.wor, L.rout = act(expect(r + "o", W, c.inner)), f32(r + "out", W)
            L.norm1 = f32(p + "norm1", W)
            if f is None:
                continue
            L.norm2 = f32(p + "norm2", W)
            if isinstance(f, MLPSpec):
                L.wup, L.wdown = act(expect(p + "mlp.up", f.ff, W)), act(expect(p + "mlp.down", W, f.ff))
                continue
            n = f.experts + f.identity
            L.wr, L.corr = f32(p + "mlp.router", n, W), f32(p + "mlp.correction", n)
            L.wup = act(torch.stack([expect(p + f"mlp.e{e}.up", f.ff, W) for e in range(f.experts)], 0))
            L.wdown = act(torch.stack([expect(p + f"mlp.e{e}.down", W, f.ff) for e in range(f.experts)], 0))
        self.layers = [own[cfg.tensor_layer(i)] for i in range(len(cfg.layers))]
        self._own = list(own.values())

    def prepare(self, max_len: int) -> None:
        """Rotary tables for positions below ``max_len`` (the engine calls this with its max_model_len before any
        step or graph capture; the design itself has no position limit)."""
        if max_len <= self._max_pos:
            return
        self._max_pos = max_len
        self._tables = {}
        for L in self.layers:
            if L.rope is not None and L.rope not in self._tables:
                self._tables[L.rope] = rope_table(max_len, L.rope[0], L.rope[1], self.device, scaling=L.rope[2])

    def param_bytes(self) -> int:
        n = 0
        for t in [self.embed, self.head] + [x for L in self._own
                                            for x in (L.wp, L.wol, L.wor, L.wx, L.wdt, L.wup, L.wdown, L.wr)]:
            if t is not None:
                n += t.numel() * t.element_size()
        return n

    # ------------------------------------------------------------------ cache and state
    def kv_bytes_per_block(self, block_size: int) -> int:
        n = 0
        for li, _, _ in self.runs:
            a = self.cfg.layers[li].mixer.left
            n += a.kv_heads * (a.dim + a.vdim)
        return max(1, n * block_size) * torch.finfo(self.dtype).bits // 8

    def allocate_kv_cache(self, num_blocks: int, block_size: int):
        """One (K [blocks, G, BS, dim], V [blocks, G, BS, vdim]) pair per layer, also where tensors are shared."""
        z = dict(dtype=self.dtype, device=self.device)
        att = [self.cfg.layers[li].mixer.left for li, _, _ in self.runs]
        return [(torch.zeros(num_blocks, a.kv_heads, block_size, a.dim, **z),
                 torch.zeros(num_blocks, a.kv_heads, block_size, a.vdim, **z)) for a in att]

    def state_bytes_per_slot(self) -> int:
        n = 0
        for li, _, _ in self.runs:
            c = self.cfg.layers[li].mixer.right
            n += c.inner * (4 * c.state + (c.taps - 1) * torch.finfo(self.dtype).bits // 8)
        return n

    def allocate_state(self, num_slots: int):
        """Per layer (the convolution's last taps - 1 inputs [slots, taps - 1, inner] in the activation type, the scan's
        fp32 state [slots, inner, state])."""
        pools = []
        for li, _, _ in self.runs:
            c = self.cfg.layers[li].mixer.right
            pools.append((torch.zeros(num_slots, c.taps - 1, c.inner, dtype=self.dtype, device=self.device),
                          torch.zeros(num_slots, c.inner, c.state, dtype=torch.float32, device=self.device)))
        return pools

    # ------------------------------------------------------------------ forward
    def _mixer(self, L, h, positions, meta: AttnMetadata, kv, state):
        """-> the two mixers' outputs [T, W] each, before their norms."""
        a, c = L.spec.mixer.left, L.spec.mixer.right
        qo, ko, vo, xo, zo = L.off
        p = linear(h, L.wp)
        kc, vc = kv
        q = rope_vnorm_store(p, qo, ko, vo, positions, self._tables[L.rope] if L.rope else None, meta.slot_mapping, kc, vc,
                             a.heads, a.kv_heads, a.dim, a.vdim, a.rot_dims, self.cfg.norm_eps, vnorm=False, bias=L.bias,
                             qw=L.qnorm, kw=L.knorm)
        left = linear(sink_attention(q, kc, vc, meta, a.scale, None, window=a.window, keep=a.keep_first), L.wol)
        cstate, sstate = state
        xc = causal_conv(p, xo, L.convw, L.convb, cstate, meta)
        y = selective_scan(xc, linear(xc, L.wx), L.wdt, c.dt_rank, L.dtb, L.A, L.skip, p, zo, sstate, meta)
        return left, linear(y, L.wor)

    def _ff(self, L, h, x):
        """-> the boundary's addends for the feed-forward of h (x: the fp32 residual, for the router)."""
        f = L.spec.mlp
        if isinstance(f, MLPSpec):
            return {"a": linear(relu2_(linear(h, L.wup)), L.wdown)}
        ids, wts, idw = moe_route(x, L.wr, f.experts + f.identity, f.top, corr=L.corr, identity=f.identity)
        return {"e": moe_experts(h, ids, L.wup, L.wdown, unit=f.unit), "ecoef": wts, "idw": idw}

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, meta: AttnMetadata, kv_caches,
                state=None, taps: list | None = None) -> torch.Tensor:
        """-> final-normed hidden [T, W].  ``state``: the pools of allocate_state (meta.state_slots names each
        sequence's slot).  ``taps``: if a list, the residual after every layer is appended."""
        if state is None or meta.state_slots is None:
            raise ValueError("this model carries recurrent state: pass state pools and meta.state_slots")
        cfg = self.cfg
        kw = dict(eps=cfg.norm_eps, mult=cfg.residual_mult, out_dtype=self.dtype)
        x = embed_gather_f32(input_ids, self.embed)
        h = postnorm_residual(x, out_dtype=self.dtype)
        for ri, (li, _, _) in enumerate(self.runs):
            L, last = self.layers[li], ri == len(self.runs) - 1
            left, right = self._mixer(L, h, positions, meta, kv_caches[ri], state[ri])
            final = self.final_norm if last else None
            h = postnorm_residual(x, left, L.lout, right, L.rout, 0.5, w=L.norm1,
                                  wn=final if L.spec.mlp is None else None, **kw)
            if L.spec.mlp is not None:
                h = postnorm_residual(x, **self._ff(L, h, x), w=L.norm2, wn=final, **kw)
            if taps is not None:
                taps.append(x.clone())
        return h if self.runs else postnorm_residual(x, wn=self.final_norm, **kw)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """final-normed hidden [B, W] -> logits [B, vocab] (a view of the padded GEMM output)."""
        return linear(hidden, self.head)[:, : self.cfg.vocab_size]
