"""Kapanex: a decoder whose sublayers run side by side on norms of their own, gated delta-rule layers between windowed
attention layers, a mixture of experts in every layer, on the paged-KV engine.

The layer list is data (models/configs.py HybridConfig, arch "kapanex").  With the fp32 residual x (the embedding row
times a constant at first) and layer norms without a bias,

    x <- x + (mixer(norm1(x)) + ff(norm2(x)))

both sublayers reading the same x.  A layer may run on another layer's tensors; its K/V cache or recurrent state is its
own.

Mixers:
  "delta"      causal convolution + SiLU over q | k | v, q and k unit vectors per head; per head an fp32 [dim, vdim] state
               that a scalar decay shrinks and a rank-one step corrects towards the token's value; the read-out is
               RMS-normed per head and gated by SiLU               [grag_causal_conv, grag_delta_scan, grag_delta_step]
  "attention"  grouped-query softmax attention in a sliding window, rotary on halves of the first rot dims, q and k
               divided by their root mean square              [grag_rope_vnorm_store with qw / kw, grag_sink_attn_*]
Feed-forward: sigmoid router scores; groups of experts ranked by their two best; the chosen scores made to sum to a
constant; SiLU-gated experts as two grouped GEMMs over the (token, expert) pairs; a shared expert under a sigmoid gate
                                                                     [grag_moe_route, grag_moe_align, grag_moe_gemm]

Per layer the mixer's input projections are one GEMM, and the layer boundary is one kernel: residual += mixer + gate *
shared + sum of weighted experts, then BOTH norms of the next layer [grag_residual_layernorm].  Activations are bf16 (or
fp32 end to end with dtype=torch.float32: the GEMMs then run in true fp32); the residual, norms, positions, angles,
scores, softmax weights, router, decays, steps, unit norms and states are fp32 in both.
"""
from __future__ import annotations

import math

import torch

from ..ops.attention import AttnMetadata, sink_attention
from ..ops.elementwise import clamped_glu, rope_table, rope_vnorm_store
from ..ops.linear import linear
from ..ops.moe import moe_experts, moe_route
from ..ops.norm import embed_gather_f32, residual_layernorm
from ..ops.recurrent import causal_conv, gated_delta
from ..parallel.comm import Group
from .configs import HybridConfig


class _Layer:
    __slots__ = ("spec", "kind", "norm1", "norm2", "wp", "off", "wo", "rope", "ones", "convw", "alog", "dtb", "onorm", "wr",
                 "wgu", "wd", "wsgu", "wsd")


def _pad8(t: torch.Tensor) -> torch.Tensor:
    """Rows padded with zeros to a multiple of 8 (projection matrices: 16-byte output rows)."""
    pad = -t.shape[0] % 8
    return t if not pad else torch.cat([t, torch.zeros(pad, *t.shape[1:], dtype=t.dtype)], 0)


def init_state_dict(cfg: HybridConfig, seed: int = 0, std: float | None = None) -> dict:
    """Random weights under the checkpoint's tensor names (bf16; benches and tests -- not a trained model)."""
    g = torch.Generator().manual_seed(seed * 1000003 + 29)
    W = cfg.hidden_size

    def r(*shape, s=None):
        s = (1.0 / math.sqrt(shape[-1])) if s is None else s
        return (torch.randn(*shape, generator=g) * (std or s)).to(torch.bfloat16)

    def around(v, n, s=0.1):
        return (v + s * torch.randn(n, generator=g)).to(torch.bfloat16)

    sd = {"embed": r(cfg.vocab_size, W, s=1.0 / max(1.0, cfg.embed_scale)), "head": r(cfg.vocab_size, W),
          "final.norm": around(1.0, W)}
    for i, L in enumerate(cfg.layers):
        if L.weights_of is not None:
            continue
        p, m, a, f = f"l{i}.", f"l{i}.mix.", L.mixer.spec, L.mlp
        sd[p + "norm1"] = around(1.0, W)
        for n, heads, dim in (("q", a.kv_heads if L.mixer.kind == "delta" else a.heads, a.dim), ("k", a.kv_heads, a.dim),
                              ("v", a.heads if L.mixer.kind == "delta" else a.kv_heads, a.vdim)):
            sd[m + n] = r(heads * dim, W)
            if L.mixer.kind == "delta":
                sd[m + n + ".conv"] = r(heads * dim, a.taps, s=0.5)
        if L.mixer.kind == "delta":
            sd.update({m + "b": r(a.heads, W), m + "a": r(a.heads, W), m + "g": r(a.heads * a.vdim, W),
                       m + "A_log": (torch.rand(a.heads, generator=g) * 2.0 - 1.5).to(torch.bfloat16),
                       m + "dt_bias": around(-3.0, a.heads, 1.0), m + "norm": around(1.0, a.vdim)})
        sd[m + "o"] = r(W, a.heads * a.vdim)
        if f is None:
            continue
        sd[p + "norm2"] = around(1.0, W)
        for e in range(f.experts):
            sd.update({p + f"mlp.e{e}.gate": r(f.ff, W), p + f"mlp.e{e}.up": r(f.ff, W), p + f"mlp.e{e}.down": r(W, f.ff)})
        sd[p + "mlp.router"] = r(f.experts, W, s=2.0 / math.sqrt(W))
        if f.shared_ff:
            sd.update({p + "mlp.shared.gate": r(f.shared_ff, W), p + "mlp.shared.up": r(f.shared_ff, W),
                       p + "mlp.shared.down": r(W, f.shared_ff), p + "mlp.shared.sg": r(1, W)})
    return sd


class KapanexModel:
    has_state = True  # recurrent state per sequence slot: the engine allocates it and never reuses cached prefixes

    def __init__(self, cfg: HybridConfig, device="cuda", dtype=torch.bfloat16, tp: Group | None = None,
                 seed: int = 0, state_dict: dict | None = None, init_std: float | None = None):
        assert cfg.arch == "kapanex", cfg.arch
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp = tp or Group([0])
        if not self.tp.trivial:
            raise NotImplementedError("the Kapanex decoder runs on one GPU per replica (no tensor parallelism)")
        if cfg.loop_stop > cfg.loop_start:
            raise ValueError("the Kapanex design has no looped layers")
        # the engine sizes the decode attention's split-KV scratch (hq * head_dim floats per row and split) and
        # picks its split plan (hkv) from these: the widest attention among the layers
        att = [L.mixer.spec for L in cfg.layers if L.mixer.kind == "attention"]
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

        def fused(*parts, pad=True):  # (name, rows) ... -> one matrix, rows fused (and padded to a multiple of 8)
            t = torch.cat([expect(n, rows, W) for n, rows in parts], 0)
            return act(_pad8(t) if pad else t)

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
            p, m = f"l{i}.", f"l{i}.mix."
            L.spec, L.kind = spec, spec.mixer.kind
            a, f = spec.mixer.spec, spec.mlp
            L.norm1 = f32(p + "norm1", W)
            H, G, vv = a.heads, a.kv_heads, a.heads * a.vdim
            if L.kind == "delta":
                qk = G * a.dim
                L.wp = fused((m + "q", qk), (m + "k", qk), (m + "v", vv), (m + "g", vv), (m + "b", H), (m + "a", H))
                conv = 2 * qk + vv
                L.off = (conv, conv + vv, conv + vv + H)  # (q | k | v from column 0) g | b | a
                L.convw = torch.cat([f32(m + "q.conv", qk, a.taps), f32(m + "k.conv", qk, a.taps),
                                     f32(m + "v.conv", vv, a.taps)], 0)
                L.alog, L.dtb = f32(m + "A_log", H), f32(m + "dt_bias", H)
                L.onorm = f32(m + "norm", a.vdim).repeat(H)  # one weight for every head
            else:
                q, k, v = H * a.dim, G * a.dim, G * a.vdim
                L.wp = fused((m + "q", q), (m + "k", k), (m + "v", v))
                L.off = (0, q, q + k)
                L.rope = (a.rot_dims, a.rot_base) if a.rot_dims else None
                # dividing by the root mean square commutes with the rotation, which keeps a head's length: the store
                # kernel norms (with a weight of ones) and then rotates, in fp32, and rounds once
                L.ones = torch.ones(a.dim, dtype=torch.float32, device=dev)
            L.wo = act(expect(m + "o", W, vv))
            if f is not None:
                f_ = p + "mlp."
                L.norm2 = f32(p + "norm2", W)
                rows = [expect(f_ + "router", f.experts, W)]
                if f.shared_ff:
                    rows.append(expect(f_ + "shared.sg", 1, W))
                    L.wsgu = fused((f_ + "shared.gate", f.shared_ff), (f_ + "shared.up", f.shared_ff), pad=False)
                    L.wsd = act(expect(f_ + "shared.down", W, f.shared_ff))
                L.wr = torch.cat(rows, 0).to(device=dev, dtype=torch.float32).contiguous()  # fp32 router (+ gate row)
                L.wgu = act(torch.stack([torch.cat([expect(f_ + f"e{e}.gate", f.ff, W), expect(f_ + f"e{e}.up", f.ff, W)], 0)
                                         for e in range(f.experts)], 0))
                L.wd = act(torch.stack([expect(f_ + f"e{e}.down", W, f.ff) for e in range(f.experts)], 0))
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
                self._tables[L.rope] = rope_table(max_len, L.rope[0], L.rope[1], self.device)

    def param_bytes(self) -> int:
        n = 0
        for t in [self.embed, self.head] + [x for L in self._own
                                            for x in (L.wp, L.wo, L.wgu, L.wd, L.wsgu, L.wsd, L.wr)]:
            if t is not None:
                n += t.numel() * t.element_size()
        return n

    # ------------------------------------------------------------------ cache and state
    def _mixers(self):
        return [self.cfg.layers[li].mixer for li, _, _ in self.runs]

    def kv_bytes_per_block(self, block_size: int) -> int:
        n = sum(m.spec.kv_heads * (m.spec.dim + m.spec.vdim) for m in self._mixers() if m.kind == "attention")
        return max(1, n * block_size) * torch.finfo(self.dtype).bits // 8

    def allocate_kv_cache(self, num_blocks: int, block_size: int):
        """One (K [blocks, G, BS, dim], V [blocks, G, BS, vdim]) pair per attention layer, also where tensors are
        shared (None for the others)."""
        z = dict(dtype=self.dtype, device=self.device)
        return [(torch.zeros(num_blocks, m.spec.kv_heads, block_size, m.spec.dim, **z),
                 torch.zeros(num_blocks, m.spec.kv_heads, block_size, m.spec.vdim, **z)) if m.kind == "attention" else None
                for m in self._mixers()]

    def state_bytes_per_slot(self) -> int:
        n = 0
        for m in self._mixers():
            a = m.spec
            if m.kind == "delta":
                n += 4 * a.heads * a.dim * a.vdim + (a.taps - 1) * a.conv_channels * torch.finfo(self.dtype).bits // 8
        return n

    def allocate_state(self, num_slots: int):
        """Per delta layer (the convolution's last taps - 1 inputs [slots, taps - 1, channels] in the activation type, an
        fp32 pool [slots, heads, dim, vdim]); attention -> None."""
        return [(torch.zeros(num_slots, m.spec.taps - 1, m.spec.conv_channels, dtype=self.dtype, device=self.device),
                 torch.zeros(num_slots, m.spec.heads, m.spec.dim, m.spec.vdim, dtype=torch.float32, device=self.device))
                if m.kind == "delta" else None for m in self._mixers()]

    # ------------------------------------------------------------------ forward
    def _mixer(self, L, h, positions, meta: AttnMetadata, kv, state):
        a, eps = L.spec.mixer.spec, self.cfg.norm_eps
        p = linear(h, L.wp)
        if L.kind == "delta":
            go, bo, ao = L.off
            cstate, sstate = state
            xc = causal_conv(p, 0, L.convw, None, cstate, meta)
            y = gated_delta(xc, p, bo, ao, go, L.alog, L.dtb, L.onorm, eps, sstate, meta, a.heads, a.kv_heads, a.dim, a.vdim)
            return linear(y, L.wo)
        qo, ko, vo = L.off
        kc, vc = kv
        q = rope_vnorm_store(p, qo, ko, vo, positions, self._tables[L.rope] if L.rope else None, meta.slot_mapping, kc, vc,
                             a.heads, a.kv_heads, a.dim, a.vdim, a.rot_dims, eps, vnorm=False, qw=L.ones, kw=L.ones)
        return linear(sink_attention(q, kc, vc, meta, a.scale, None, window=a.window), L.wo)

    def _ff(self, L, h):
        """-> the boundary's feed-forward addends: shared output and its gate, experts' outputs and their weights."""
        f = L.spec.mlp
        ids, wts, sgate = moe_route(h, L.wr, f.experts, f.top, f.groups, f.keep, score=f.score, group_top=f.group_top,
                                    scale=f.scale)
        add = {"e": moe_experts(h, ids, L.wgu, L.wd), "ecoef": wts}
        if L.wsgu is not None:
            add.update(b=linear(clamped_glu(linear(h, L.wsgu), None, 1.0, 0.0), L.wsd), bcoef=sgate)
        return add

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, meta: AttnMetadata, kv_caches,
                state=None, taps: list | None = None) -> torch.Tensor:
        """-> final-normed hidden [T, W].  ``state``: the pools of allocate_state (meta.state_slots names each
        sequence's slot).  ``taps``: if a list, the residual after every layer is appended."""
        if state is None or meta.state_slots is None:
            raise ValueError("this model carries recurrent state: pass state pools and meta.state_slots")
        kw = dict(eps=self.cfg.norm_eps, out_dtype=self.dtype)
        x = embed_gather_f32(input_ids, self.embed, self.cfg.embed_scale)
        pend = {}  # the previous layer's outputs, added at the next boundary
        for ri, (li, _, _) in enumerate(self.runs):
            L = self.layers[li]
            h1, h2 = residual_layernorm(x, L.norm1, L.norm2, **pend, **kw)
            if taps is not None and ri:
                taps.append(x.clone())
            pend = {"a": self._mixer(L, h1, positions, meta, kv_caches[ri], state[ri])}
            if L.wr is not None:
                pend.update(self._ff(L, h2))
        h, _ = residual_layernorm(x, self.final_norm, **pend, **kw)
        if taps is not None and self.runs:
            taps.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """final-normed hidden [B, W] -> logits [B, vocab] (a view of the padded GEMM output)."""
        return linear(hidden, self.head)[:, : self.cfg.vocab_size]
