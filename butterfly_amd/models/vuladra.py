"""Vuladra: a decoder-only LM whose sublayers sit between two RMS norms (ModelConfig.layer_specs).

  embedding   : x = table[token], an f32 residual
  every layer : x <- x + rms_1b(mixer(rms_1(x))), then x <- x + rms_2b(ff(rms_2(x)))
    mixer "pooled_attention" : GQA without rotation; queries and keys RMS-normed over the whole projection
                        (all heads together); a visible key weighs in with sigmoid(score + a number per
                        head), not normalised over the keys; visible are the tokens of a sliding window
                        and, wholly before it, blocks of `pool` tokens through their mean key and value;
                        an elementwise sigmoid gate before the output projection
    mixer "side_by_side"     : two mixers on the same input, summed with a constant factor each: windowed
                        softmax GQA without rotation, and linear attention on silu'd q, k, v whose state
                        decays by a constant per head, RMS-normed over all heads, sigmoid-gated
    mixer "selective_scan"   : input-dependent state-space recurrence per channel: short causal convolution
                        with bias + silu, step sizes through a low-rank projection and softplus, a skip,
                        a silu gate
    feed-forward      : dense silu GLU, or the top experts by router logit (f32, softmax over the chosen
                        logits) plus a shared expert, all clamped GLUs g sigmoid(1.702 g) (u + 1)
  output      : RMS norm, logits = table x, f32

Every size and constant comes from the config; the residual, norms, scores and weights, step sizes,
decays and recurrent states are f32 in the bf16 model too. Unsharded (tp = pp = ep = 1). Prompt chunks
always attend through the paged cache, so one attention op serves fresh prompts, continuation chunks
and decoded tokens. The mean keys and values of pooled blocks are kept with the page in which the
block ends, so they are handed out, shared, reused and freed with the pages; the recurrent states and
the convolutions' last inputs live in the cache's per-sequence state slots.
"""
from __future__ import annotations

import math
from typing import Optional

import torch

from .. import ops
from ..config import ModelConfig
from ..engine.batch import ForwardBatch
from ..parallel.comm import Communicator
from .shard import LocalDims, Shard
from .stack import PackedStack, pad128
from .transformer import LogicalParam, _name_seed

EXPERT_ALPHA, EXPERT_UP_OFFSET = 1.702, 1.0      # routed and shared experts: g sigmoid(alpha g) (u + offset)
NO_WINDOW = 1 << 30                              # plain causal attention


class VuladraLM(PackedStack):
    attention_types = ("pooled_attention", "side_by_side")

    def __init__(self, cfg: ModelConfig, shard: Shard = Shard(), device="cpu",
                 dtype: torch.dtype = torch.bfloat16, comm: Optional[Communicator] = None):
        if not cfg.layer_specs:
            raise ValueError("Vuladra needs ModelConfig.layer_specs (ModelConfig.from_vuladra)")
        if shard.tp_size != 1 or shard.ep_size != 1 or shard.layer_start != 0 or \
                (shard.layer_end is not None and shard.layer_end != cfg.num_layers):
            raise NotImplementedError("Vuladra runs unsharded (tp = pp = ep = 1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Vuladra runs in bfloat16 or float32")
        for sp in cfg.layer_specs:
            if sp["type"] not in self.attention_types + ("selective_scan",):
                raise ValueError(f"layer {sp['index']}: Vuladra has no mixer {sp['type']!r}")
        self.cfg, self.shard = cfg, shard
        self.device, self.dtype = torch.device(device), dtype
        self.comm = comm or Communicator.single()
        self.specs = cfg.layer_specs
        self.layer_ids = list(range(cfg.num_layers))
        self.first = self.last = True
        self.tp = self.ep = 1
        vpad = pad128(cfg.vocab_size)
        self.dims = LocalDims(hq=max(cfg.num_heads, 1), hkv=cfg.num_kv_heads, kv_head0=0, q_head0=0,
                              ffn=max(cfg.intermediate_size, 1), ffn0=0, vocab=vpad, vocab0=0, vocab_padded=vpad,
                              experts=max(cfg.num_experts, 1), expert0=0)
        # layer -> index of its cache tuple / of its first state tensor, and its cached head sizes (padded
        # with zeros to sizes the attention's matrix-core form tiles)
        self.cache_index, self.state_index, self.cache_dims = {}, {}, {}
        n = 0
        for sp in self.specs:
            i = sp["index"]
            if sp["type"] in self.attention_types:
                self.cache_index[i] = len(self.cache_index)
                self.cache_dims[i] = (ops.attn_window_pad(sp["dim"], dtype), ops.attn_window_pad(sp["vdim"], dtype))
            if sp["type"] != "pooled_attention":
                self.state_index[i] = n
                n += 1 if sp["type"] == "side_by_side" else 2
        self.has_state = bool(self.state_index)
        self.state: list = []                     # set by allocate_state (the cache object owns the pool)
        self.layer_probe = None                   # debug hook: f(layer, residual [T, W] f32) after every layer
        self.p: dict[str, torch.Tensor] = {}
        self.packed: dict = {}
        self._arange: dict = {}
        self._alloc()

    # ------------------------------------------------------------------------------------
    # parameters
    # ------------------------------------------------------------------------------------
    @staticmethod
    def _mixer_rows(sp) -> list:
        """(tensor name, rows) of the mixer's input projections in the order they are fused."""
        H, G, D, Dv = sp["heads"], sp["kv_heads"], sp["dim"], sp["vdim"]
        if sp["type"] == "pooled_attention":
            return [("q", H * D), ("k", G * D), ("v", G * Dv), ("g", H * Dv)]
        if sp["type"] == "side_by_side":
            h, d, dv = sp["r_heads"], sp["r_dim"], sp["r_vdim"]
            return [("left.q", H * D), ("left.k", G * D), ("left.v", G * Dv), ("right.q", h * d), ("right.k", h * d),
                    ("right.v", h * dv), ("right.g", h * dv)]
        return [("in", 2 * sp["inner"])]

    def _alloc(self):
        c, W = self.cfg, self.cfg.hidden_size
        z = lambda *s: torch.zeros(*s, dtype=self.dtype, device=self.device)                  # noqa: E731
        f = lambda *s: torch.zeros(*s, dtype=torch.float32, device=self.device)               # noqa: E731
        p = self.p

        p["embed"] = z(self.dims.vocab, W)             # also the LM head; rows past the vocabulary stay zero
        for sp in self.specs:
            pre = f"l{sp['index']}."
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if sp["ffn"] else ()):
                p[pre + n] = f(W)
            H, G, D, Dv = sp["heads"], sp["kv_heads"], sp["dim"], sp["vdim"]
            p[pre + "in"] = z(self._wide(sum(r for _, r in self._mixer_rows(sp)), W), W)
            if sp["type"] == "pooled_attention":
                p[pre + "q.norm"], p[pre + "k.norm"], p[pre + "pb"] = f(H * D), f(G * D), f(H)
                p[pre + "o"] = z(W, H * Dv)
            elif sp["type"] == "side_by_side":
                p[pre + "norm"] = f(sp["r_heads"] * sp["r_vdim"])
                p[pre + "decay"] = ops.decay_powers(sp["decay"], self.device)
                p[pre + "inv_freq"] = f(0)                                        # (no rotation)
                # one output projection of [left heads | right heads]
                p[pre + "o"] = z(W, H * Dv + sp["r_heads"] * sp["r_vdim"])
            else:
                C, N, R = sp["inner"], sp["state"], sp["dt_rank"]
                p[pre + "conv"], p[pre + "conv.b"] = f(C, sp["taps"]), f(C)
                p[pre + "x"], p[pre + "dt"] = z(self._wide(R + 2 * N, C), C), z(C, R)
                p[pre + "dt.b"], p[pre + "A_log"], p[pre + "D"] = f(C), f(C, N), f(C)
                p[pre + "o"] = z(W, C)
            fs = sp["ffn"]
            if fs and fs["kind"] == "dense":
                self._glu_alloc(pre, fs["ff"], float("inf"), 1.0, 0.0)
            elif fs:
                E, F = fs["experts"], fs["ff"]
                p[pre + "router"] = z(E, W)
                p[pre + "experts.gate_up"], p[pre + "experts.down"] = z(E, 2 * F, W), z(E, W, F)
                if fs["shared"]:
                    self._glu_alloc(pre + "shared.", fs["shared"]["ff"], fs["shared"]["limit"], EXPERT_ALPHA, EXPERT_UP_OFFSET)
        p["final.norm"] = f(W)

    @property
    def head_weight(self) -> torch.Tensor:
        return self.p["embed"]

    def logical_params(self) -> list[LogicalParam]:
        """Checkpoint tensors by their file names ('l<i>.mix.q', 'l<i>.mlp.e<j>.up', ...), each a view into
        the fused local tensors."""
        c, p = self.cfg, self.p
        out: list[LogicalParam] = []

        def add(name, t, init="normal", put=None, shape=None, get=None):
            out.append(LogicalParam(name, tuple(shape or t.shape), None, 0, 0, init, get or (lambda t=t: t),
                                    put or (lambda x, t=t: t.copy_(x.reshape(t.shape)))))

        add("embed", p["embed"][:c.vocab_size], "embed")
        for sp in self.specs:
            L = f"l{sp['index']}."
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if sp["ffn"] else ()):
                add(L + n, p[L + n], "ones")
            at = 0
            for n, rows in self._mixer_rows(sp):
                add(L + "mix." + n, p[L + "in"][at:at + rows])
                at += rows
            if sp["type"] == "pooled_attention":
                add(L + "mix.q.norm", p[L + "q.norm"], "ones")
                add(L + "mix.k.norm", p[L + "k.norm"], "ones")
                add(L + "mix.pb", p[L + "pb"], "key_bias")
                add(L + "mix.o", p[L + "o"])
            elif sp["type"] == "side_by_side":
                nl = sp["heads"] * sp["vdim"]
                add(L + "mix.right.norm", p[L + "norm"], "ones")
                add(L + "mix.left.o", p[L + "o"][:, :nl])
                add(L + "mix.right.o", p[L + "o"][:, nl:])
            else:
                add(L + "mix.conv", p[L + "conv"], "taps")
                add(L + "mix.conv.b", p[L + "conv.b"], "small")
                add(L + "mix.x", p[L + "x"][:sp["dt_rank"] + 2 * sp["state"]])
                add(L + "mix.dt", p[L + "dt"])
                add(L + "mix.dt.b", p[L + "dt.b"], "dt_bias")
                add(L + "mix.A_log", p[L + "A_log"], "a_log")
                add(L + "mix.D", p[L + "D"], "ones")
                add(L + "mix.o", p[L + "o"])
            fs = sp["ffn"]
            if fs and fs["kind"] == "dense":
                self._glu_logical(add, L + "mlp.", L, fs["ff"])
            elif fs:
                F = fs["ff"]
                add(L + "mlp.router", p[L + "router"])
                for e in range(fs["experts"]):
                    add(L + f"mlp.e{e}.gate", p[L + "experts.gate_up"][e, :F])
                    add(L + f"mlp.e{e}.up", p[L + "experts.gate_up"][e, F:])
                    add(L + f"mlp.e{e}.down", p[L + "experts.down"][e])
                if fs["shared"]:
                    self._glu_logical(add, L + "mlp.shared.", L + "shared.", fs["shared"]["ff"])
        add("final.norm", p["final.norm"], "ones")
        return out

    @torch.no_grad()
    def init_random(self, seed: int = 0) -> None:
        """Deterministic random weights: each tensor is drawn on the host from a generator keyed on
        (seed, tensor name). Projections are scaled by 1 / sqrt(fan-in), the embedding has unit entries,
        norm weights sit around one, a channel's n-th state decays about n times as fast as its first,
        step sizes lie well below one, key biases such that far keys weigh little."""
        for lp in self.logical_params():
            g = torch.Generator().manual_seed(_name_seed(lp.name, seed))
            shp = lp.global_shape
            r = torch.randn(shp, generator=g)
            if lp.init == "normal":
                t = r / math.sqrt(shp[-1])
            elif lp.init == "embed":
                t = r
            elif lp.init == "ones":
                t = 1.0 + 0.1 * r
            elif lp.init == "small":
                t = 0.1 * r
            elif lp.init == "taps":
                t = 0.5 * r
            elif lp.init == "key_bias":
                t = -3.0 + 0.5 * r
            elif lp.init == "dt_bias":
                t = -3.0 + r
            elif lp.init == "a_log":
                t = torch.log(torch.arange(1, shp[1] + 1).float())[None] + 0.1 * r
            else:
                raise ValueError(lp.init)
            # weights are bf16 values in every run (an f32 model holds them exactly)
            lp.set(t.to(torch.bfloat16).to(self.device))

    # ------------------------------------------------------------------------------------
    # caches
    # ------------------------------------------------------------------------------------
    def kv_bytes_per_token(self, dtype: Optional[torch.dtype] = None) -> int:
        es = torch.empty((), dtype=dtype or self.dtype).element_size()
        n = 0
        for i in self.cache_index:
            sp, (dk, dv) = self.specs[i], self.cache_dims[i]
            # pooled rows: one per `pool` tokens, rounded up per page of 32 tokens
            n += sp["kv_heads"] * (dk + dv) * es * (32 + (ops.pool_rows(32, sp["pool"]) if sp["pool"] else 0)) / 32
        return max(1, math.ceil(n))

    def state_bytes_per_slot(self) -> int:
        n = 0
        for i in self.state_index:
            sp = self.specs[i]
            n += sp["r_heads"] * sp["r_dim"] * sp["r_vdim"] if sp["type"] == "side_by_side" \
                else sp["inner"] * (sp["taps"] - 1 + sp["state"])
        return 4 * n

    def allocate_kv_cache(self, num_blocks: int, block_size: int, dtype: Optional[torch.dtype] = None) -> list:
        """One (K [blocks, G, BS, D], V [blocks, G, Dv, BS]) pair per attention layer, V with a page's tokens
        contiguous, head sizes padded with zeros; a layer with pooled blocks has their mean keys and
        values [blocks, G, rows per page, D or Dv] behind the pair."""
        dt = dtype or self.dtype
        if dt != self.dtype:
            raise NotImplementedError("Vuladra caches hold the model's element type")
        caches = []
        for i in self.cache_index:
            sp, (dk, dv) = self.specs[i], self.cache_dims[i]
            shapes = [(block_size, dk), (dv, block_size)]
            if sp["pool"]:
                n = ops.pool_rows(block_size, sp["pool"])
                shapes += [(n, dk), (n, dv)]
            caches.append(tuple(torch.zeros(num_blocks, sp["kv_heads"], *s, dtype=dt, device=self.device) for s in shapes))
        return caches

    def allocate_state(self, num_slots: int) -> list:
        """f32 tensors per recurrent layer: side by side, the linear attention's matrices [slots, H, D, Dv];
        selective scan, the last taps - 1 convolution inputs [slots, taps - 1, C] (oldest first) and the
        states [slots, C, N]."""
        f = lambda *s: torch.zeros(num_slots, *s, dtype=torch.float32, device=self.device)     # noqa: E731
        self.state = []
        for i in self.state_index:
            sp = self.specs[i]
            if sp["type"] == "side_by_side":
                self.state.append(f(sp["r_heads"], sp["r_dim"], sp["r_vdim"]))
            else:
                self.state += [f(sp["taps"] - 1, sp["inner"]), f(sp["inner"], sp["state"])]
        return self.state

    # ------------------------------------------------------------------------------------
    # forward
    # ------------------------------------------------------------------------------------
    def forward(self, fb: ForwardBatch, kv_caches: Optional[list] = None,
                hidden_in: Optional[torch.Tensor] = None) -> torch.Tensor:
        """One step over the packed rows of `fb`; returns f32 logits [R, padded vocab] for the rows
        fb.logits_idx names (None: all)."""
        p, eps = self.p, self.cfg.norm_eps
        meta = self._step_meta(fb)
        meta["one_row"] = not fb.is_prefill        # decoding: every sequence of the step has one row
        if self.has_state and fb.num_tokens and not self.state:
            raise RuntimeError("Vuladra: the recurrent-state pool is not allocated (KVCache state slots)")
        if kv_caches is None and self.cache_index:
            raise RuntimeError("Vuladra attention runs through the paged cache")
        x = ops.embed_scaled(fb.input_ids, p["embed"], 1.0)
        # sublayers in order: (layer, 1 = mixer / 2 = feed-forward)
        subs = [(sp, q) for sp in self.specs for q in ((1, 2) if sp["ffn"] else (1,))]
        h = ops.par_final(x, None, None, p[f"l{subs[0][0]['index']}.norm1"], eps, 0.0, None, self.dtype) if subs else None
        for n, (sp, q) in enumerate(subs):
            i = sp["index"]
            pre = f"l{i}."
            if q == 2:
                y = self._ffn(sp["ffn"], pre, h)
            elif sp["type"] == "pooled_attention":
                y = self._pooled_attention(sp, pre, h, fb, meta, kv_caches[self.cache_index[i]])
            elif sp["type"] == "side_by_side":
                y = self._side_by_side(sp, pre, h, fb, meta, kv_caches[self.cache_index[i]])
            else:
                y = self._selective_scan(sp, pre, h, fb, meta)
            nxt = subs[n + 1] if n + 1 < len(subs) else None
            # the residual update fused with the next sublayer's norm
            h = ops.post_norm_add_norm(x, y, p[pre + f"norm{q}b"], None, eps, 1.0, None,
                                       p[f"l{nxt[0]['index']}.norm{nxt[1]}"] if nxt else None, None, self.dtype, rms=True)
            if self.layer_probe is not None and (nxt is None or nxt[1] == 1):
                self.layer_probe(i, x)
        xf = ops.par_final(x, None, None, p["final.norm"], eps, 0.0, fb.logits_idx, self.dtype)
        return ops.linear_act(xf, p["embed"], out_dtype=torch.float32)

    def _pooled_attention(self, sp, pre, h, fb, meta, cache):
        T, p = fb.num_tokens, self.p
        H, G, D, Dv = sp["heads"], sp["kv_heads"], sp["dim"], sp["vdim"]
        kc, vc = cache[:2]
        pool = (sp["pool"], cache[2], cache[3]) if sp["pool"] else None
        z = ops.linear_act(h, p[pre + "in"])
        o1, o2 = H * D, H * D + G * D
        o3 = o2 + G * Dv
        q, k, v = z[:, :o1].view(T, H, D), z[:, o1:o2].view(T, G, D), z[:, o2:o3].view(T, G, Dv)
        qp = ops.qk_norm_rows_kv(q, k, v, p[pre + "q.norm"], p[pre + "k.norm"], self.cfg.norm_eps, fb.positions, fb.slots,
                                 kc, vc, pool, meta["tables"], meta["row_cu"], meta["row_map"], meta["one_row"])
        o = ops.attn_window_paged(qp, kc, vc, meta["tables"], meta["row_cu"], fb.positions, sp["scale"],
                                  min(sp["window"], NO_WINDOW), 0, None, row_map=meta["row_map"], sigmoid=True,
                                  key_bias=p[pre + "pb"], pool=pool, gate=z[:, o3:o3 + H * Dv], dv_out=Dv)
        return ops.linear_act(o, p[pre + "o"])

    def _side_by_side(self, sp, pre, h, fb, meta, cache):
        T, p, eps = fb.num_tokens, self.p, self.cfg.norm_eps
        H, G, D, Dv = sp["heads"], sp["kv_heads"], sp["dim"], sp["vdim"]
        kc, vc = cache
        z = ops.linear_act(h, p[pre + "in"])
        cut = [0]
        for _, rows in self._mixer_rows(sp):
            cut.append(cut[-1] + rows)
        part = lambda j, heads: z[:, cut[j]:cut[j + 1]].view(T, heads, -1)                     # noqa: E731
        # both halves leave their heads, times their factor, in one row: [left | right]
        y = ops.new_empty(T, p[pre + "o"].shape[1], dtype=self.dtype, device=self.device)
        nl = H * Dv
        qp = ops.qk_norm_rope_kv(part(0, H), part(1, G), part(2, G), None, None, eps, fb.positions, p[pre + "inv_freq"],
                                 fb.slots, kc, vc)
        ops.attn_window_paged(qp, kc, vc, meta["tables"], meta["row_cu"], fb.positions, sp["scale"],
                              min(sp["window"], NO_WINDOW), 0, None, row_map=meta["row_map"], out_mul=sp["left_scale"],
                              dv_out=Dv, out=y[:, :nl])
        h2 = sp["r_heads"]
        o = ops.decay_scan(part(3, h2), part(4, h2), part(5, h2), p[pre + "decay"], self.state[self.state_index[sp["index"]]],
                           meta["state_slots"], meta["row_cu"], fb.positions, "silu", meta["one_row"])
        ops.row_norm_gate(o.view(T, -1), p[pre + "norm"], eps, z[:, cut[6]:cut[7]], sp["right_scale"], y[:, nl:])
        return ops.linear_act(y, p[pre + "o"])

    def _selective_scan(self, sp, pre, h, fb, meta):
        p, si = self.p, self.state_index[sp["index"]]
        C, N, R = sp["inner"], sp["state"], sp["dt_rank"]
        u = ops.linear_act(h, p[pre + "in"])
        x = ops.short_conv_step(u[:, :C], p[pre + "conv"], self.state[si], meta["state_slots"], meta["row_cu"], fb.positions,
                                "silu", self.dtype, p[pre + "conv.b"], meta["one_row"])
        s = ops.linear_act(x, p[pre + "x"])                                     # dt | B | C
        y = ops.selective_scan(x, s[:, :R], p[pre + "dt"], s[:, R:R + N], s[:, R + N:R + 2 * N], u[:, C:2 * C],
                               p[pre + "A_log"], p[pre + "dt.b"], p[pre + "D"], self.state[si + 1], meta["state_slots"],
                               meta["row_cu"], fb.positions, meta["one_row"])
        return ops.linear_act(y, p[pre + "o"])

    def _ffn(self, fs, pre, h):
        p = self.p
        if fs["kind"] == "dense":
            return self._glu(pre, h, fs["ff"], float("inf"), 1.0, 0.0).contiguous()
        sh = fs["shared"]
        add = self._glu(pre + "shared.", h, sh["ff"], sh["limit"], EXPERT_ALPHA, EXPERT_UP_OFFSET) if sh else None
        ids, w = ops.moe_route_scores(h, p[pre + "router"], fs["top"], scoring="softmax", renorm=True)
        return ops.moe_glu_ffn(h, ids, w, p[pre + "experts.gate_up"], p[pre + "experts.down"], fs["limit"], EXPERT_ALPHA,
                               up_offset=EXPERT_UP_OFFSET, scale_input=False, addend=add)
