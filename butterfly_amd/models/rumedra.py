"""Rumedra: a decoder-only pre-norm LM of two mixers (ModelConfig.layer_specs).

  embedding   : x = table[token] * scale, an f32 residual
  every layer : x <- x + mixer(rms_1(x)), then x <- x + ff(rms_2(x))
    mixer "attention_retention" : two mixers on the same input, summed with a constant factor each. Left: GQA
                        with biases, half-rotated queries and keys on the first dims (frequencies optionally
                        rescaled by wavelength), a sliding window, an ordinary softmax, an elementwise sigmoid
                        gate. Right: linear attention with one constant decay per head (retention), queries
                        and keys half-rotated, keys times dim^(-1/2), unit RMS per head, a silu gate
    mixer "hgrn"      : linear attention with a decay per channel f = l + (1 - l) sigmoid(W_f h + b) and the key
                        1 - f, S <- diag(f) S + (1 - f) v^T, o = S^T silu(q), RMS norm per head
    feed-forward      : dense ReLU GLU, or routed silu GLUs: f32 softmax scores, chosen with a correction among
                        the best groups of experts, identity experts that hand on their input, a shared expert
  output      : RMS norm, logits = table x, f32

Every size and constant comes from the config; the residual, norms, scores and softmax, rotations, gates and
decays of the recurrences and their states are f32 in the bf16 model too. Unsharded (tp = pp = ep = 1). Prompt
chunks always attend through the paged cache, so one attention op serves fresh prompts, continuation chunks and
decoded tokens; the recurrent states live in the cache's per-sequence state slots.
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

NO_LIMIT = float("inf")             # the GLUs are not clamped
RELU, SILU = float("inf"), 1.0      # g sigmoid(alpha g): the dense feed-forward's gate, the experts' gate
RENORM_EPS = 1e-20                  # added to the sum that divides the chosen scores
NO_WINDOW = 1 << 30


class RumedraLM(PackedStack):
    attention_types = ("attention_retention",)

    def __init__(self, cfg: ModelConfig, shard: Shard = Shard(), device="cpu",
                 dtype: torch.dtype = torch.bfloat16, comm: Optional[Communicator] = None):
        if not cfg.layer_specs:
            raise ValueError("Rumedra needs ModelConfig.layer_specs (ModelConfig.from_rumedra)")
        if shard.tp_size != 1 or shard.ep_size != 1 or shard.layer_start != 0 or \
                (shard.layer_end is not None and shard.layer_end != cfg.num_layers):
            raise NotImplementedError("Rumedra runs unsharded (tp = pp = ep = 1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Rumedra runs in bfloat16 or float32")
        for sp in cfg.layer_specs:
            if sp["type"] not in self.attention_types + ("hgrn",):
                raise ValueError(f"layer {sp['index']}: Rumedra has no mixer {sp['type']!r}")
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
        # layer -> index of its cache pair, and its cached head sizes (padded with zeros to sizes the attention's
        # matrix-core form tiles); every layer has one state tensor
        self.cache_index, self.cache_dims = {}, {}
        for sp in self.specs:
            if sp["type"] in self.attention_types:
                self.cache_index[sp["index"]] = len(self.cache_index)
                self.cache_dims[sp["index"]] = (ops.attn_window_pad(sp["dim"], dtype), ops.attn_window_pad(sp["vdim"], dtype))
        self.has_state = bool(self.specs)
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
        h, d, dv = sp["r_heads"], sp["r_dim"], sp["r_vdim"]
        if sp["type"] == "hgrn":
            return [("q", h * d), ("f", h * d), ("v", h * dv)]
        H, G, D, Dv = sp["heads"], sp["kv_heads"], sp["dim"], sp["vdim"]
        return [("left.q", H * D), ("left.k", G * D), ("left.v", G * Dv), ("left.g", H * Dv),
                ("right.q", h * d), ("right.k", h * d), ("right.v", h * dv), ("right.g", h * dv)]

    def _alloc(self):
        c, W = self.cfg, self.cfg.hidden_size
        z = lambda *s: torch.zeros(*s, dtype=self.dtype, device=self.device)                  # noqa: E731
        f = lambda *s: torch.zeros(*s, dtype=torch.float32, device=self.device)               # noqa: E731
        p = self.p
        p["embed"] = z(self.dims.vocab, W)             # also the LM head; rows past the vocabulary stay zero
        for sp in self.specs:
            pre = f"l{sp['index']}."
            for n in ("norm1",) + (("norm2",) if sp["ffn"] else ()):
                p[pre + n] = f(W)
            h, d, dv = sp["r_heads"], sp["r_dim"], sp["r_vdim"]
            rows = self._wide(sum(r for _, r in self._mixer_rows(sp)), W)
            p[pre + "in"] = z(rows, W)
            if sp["type"] == "hgrn":
                p[pre + "f.b"], p[pre + "lower"], p[pre + "norm"] = f(h * d), f(h * d), f(dv)
                no = h * dv
            else:
                p[pre + "in.b"] = z(rows)                        # biases of the left q, k, v; zeros elsewhere
                p[pre + "decay"] = ops.decay_powers(sp["decay"], self.device)
                for side in ("", "r_"):
                    inv = ops.rope_inv_freq(sp[side + "rot_dims"], sp[side + "rot_base"], sp[side + "rot_scaling"])
                    p[pre + side + "inv_freq"] = inv.to(torch.float32).to(self.device)
                # one output projection of [left heads | right heads]
                no = sp["heads"] * sp["vdim"] + h * dv
            p[pre + "o"] = z(self._wide(W, no), no)
            fs = sp["ffn"]
            if fs and fs["kind"] == "dense":
                self._glu_alloc(pre, fs["ff"], NO_LIMIT, RELU, 0.0)
            elif fs:
                E, F = fs["experts"], fs["ff"]
                p[pre + "router"], p[pre + "correction"] = z(E + fs["identity"], W), f(E + fs["identity"])
                p[pre + "experts.gate_up"], p[pre + "experts.down"] = z(E, 2 * F, W), z(E, W, F)
                if fs["shared"]:
                    self._glu_alloc(pre + "shared.", fs["shared"]["ff"], NO_LIMIT, SILU, 0.0)
        p["final.norm"] = f(W)

    @property
    def head_weight(self) -> torch.Tensor:
        return self.p["embed"]

    def logical_params(self) -> list[LogicalParam]:
        """Checkpoint tensors by their file names ('l<i>.mix.left.q', 'l<i>.mlp.e<j>.up', ...), each a view into
        the fused local tensors."""
        c, p = self.cfg, self.p
        W = c.hidden_size
        out: list[LogicalParam] = []

        def add(name, t, init="normal", put=None, shape=None, get=None):
            out.append(LogicalParam(name, tuple(shape or t.shape), None, 0, 0, init, get or (lambda t=t: t),
                                    put or (lambda x, t=t: t.copy_(x.reshape(t.shape)))))

        add("embed", p["embed"][:c.vocab_size], "embed")
        for sp in self.specs:
            L = f"l{sp['index']}."
            for n in ("norm1",) + (("norm2",) if sp["ffn"] else ()):
                add(L + n, p[L + n], "ones")
            at = 0
            for n, rows in self._mixer_rows(sp):
                add(L + "mix." + n, p[L + "in"][at:at + rows])
                if n in ("left.q", "left.k", "left.v"):
                    add(L + f"mix.{n}.b", p[L + "in.b"][at:at + rows], "small")
                at += rows
            if sp["type"] == "hgrn":
                add(L + "mix.f.b", p[L + "f.b"], "forget_bias")
                add(L + "mix.lower", p[L + "lower"], "lower")
                add(L + "mix.norm", p[L + "norm"], "ones")
                add(L + "mix.o", p[L + "o"][:W])
            else:
                nl = sp["heads"] * sp["vdim"]
                add(L + "mix.left.o", p[L + "o"][:W, :nl])
                add(L + "mix.right.o", p[L + "o"][:W, nl:])
            fs = sp["ffn"]
            if fs and fs["kind"] == "dense":
                self._glu_logical(add, L + "mlp.", L, fs["ff"])
            elif fs:
                F = fs["ff"]
                add(L + "mlp.router", p[L + "router"])
                add(L + "mlp.correction", p[L + "correction"], "small")
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
        (seed, tensor name). Projections are scaled by 1 / sqrt(fan-in), the embedding has unit entries, norm
        weights sit around one, forget gates well above their lower bounds."""
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
            elif lp.init == "forget_bias":
                t = 2.0 + r
            elif lp.init == "lower":
                t = torch.sigmoid(r) * 0.9
            else:
                raise ValueError(lp.init)
            # weights are bf16 values in every run (an f32 model holds them exactly)
            lp.set(t.to(torch.bfloat16).to(self.device))

    # ------------------------------------------------------------------------------------
    # caches
    # ------------------------------------------------------------------------------------
    def kv_bytes_per_token(self, dtype: Optional[torch.dtype] = None) -> int:
        es = torch.empty((), dtype=dtype or self.dtype).element_size()
        return max(1, es * sum(self.specs[i]["kv_heads"] * sum(self.cache_dims[i]) for i in self.cache_index))

    def state_bytes_per_slot(self) -> int:
        return sum(4 * sp["r_heads"] * sp["r_dim"] * sp["r_vdim"] for sp in self.specs)

    def allocate_kv_cache(self, num_blocks: int, block_size: int, dtype: Optional[torch.dtype] = None) -> list:
        """One (K [blocks, G, BS, D], V [blocks, G, Dv, BS]) pair per attention layer, V with a page's tokens
        contiguous, head sizes padded with zeros."""
        dt = dtype or self.dtype
        if dt != self.dtype:
            raise NotImplementedError("Rumedra caches hold the model's element type")
        z = lambda *s: torch.zeros(*s, dtype=dt, device=self.device)                          # noqa: E731
        return [(z(num_blocks, self.specs[i]["kv_heads"], block_size, self.cache_dims[i][0]),
                 z(num_blocks, self.specs[i]["kv_heads"], self.cache_dims[i][1], block_size)) for i in self.cache_index]

    def allocate_state(self, num_slots: int) -> list:
        """One f32 tensor per layer: its linear attention's matrices [slots, H, D, Dv]."""
        self.state = [torch.zeros(num_slots, sp["r_heads"], sp["r_dim"], sp["r_vdim"], dtype=torch.float32, device=self.device)
                      for sp in self.specs]
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
        meta["rope"] = {}                          # rotation tables of the step, by their frequencies
        if self.has_state and fb.num_tokens and not self.state:
            raise RuntimeError("Rumedra: the recurrent-state pool is not allocated (KVCache state slots)")
        if kv_caches is None and self.cache_index:
            raise RuntimeError("Rumedra attention runs through the paged cache")
        x = ops.embed_scaled(fb.input_ids, p["embed"], self.cfg.embed_scale)
        # sublayers in order: (layer, 1 = mixer / 2 = feed-forward)
        subs = [(sp, q) for sp in self.specs for q in ((1, 2) if sp["ffn"] else (1,))]
        h = ops.par_final(x, None, None, p[f"l{subs[0][0]['index']}.norm1"], eps, 0.0, None, self.dtype) if subs else None
        y = None
        for n, (sp, q) in enumerate(subs):
            i = sp["index"]
            pre = f"l{i}."
            if q == 2:
                y = self._ffn(sp["ffn"], pre, h)
            elif sp["type"] == "hgrn":
                y = self._hgrn(sp, pre, h, fb, meta)
            else:
                y = self._attention_retention(sp, pre, h, fb, meta, kv_caches[self.cache_index[i]])
            nxt = subs[n + 1] if n + 1 < len(subs) else None
            if nxt:      # the residual update fused with the next sublayer's norm
                h = ops.add_norm(x, y, p[f"l{nxt[0]['index']}.norm{nxt[1]}"], eps, self.dtype)
            if self.layer_probe is not None and (nxt is None or nxt[1] == 1):
                self.layer_probe(i, x if nxt else x + y.float())
        # the last update fused with the output norm, on the rows that are asked for
        xf = ops.par_final(x, y, None, p["final.norm"], eps, 0.0, fb.logits_idx, self.dtype)
        return ops.linear_act(xf, p["embed"], out_dtype=torch.float32)

    def _rope(self, name, fb, meta, *spec):
        if spec not in meta["rope"]:
            meta["rope"][spec] = ops.rope_table(fb.positions, self.p[name])
        return meta["rope"][spec]

    def _out(self, y, w):
        """Output projection (its rows may be padded)."""
        y, W = ops.linear_act(y, w), self.cfg.hidden_size
        return y if y.shape[1] == W else y[:, :W].contiguous()

    def _attention_retention(self, sp, pre, h, fb, meta, cache):
        T, p, eps = fb.num_tokens, self.p, self.cfg.norm_eps
        z = ops.linear_act(h, p[pre + "in"], bias=p[pre + "in.b"])
        cut = [0]
        for _, rows in self._mixer_rows(sp):
            cut.append(cut[-1] + rows)
        part = lambda j, heads: z[:, cut[j]:cut[j + 1]].view(T, heads, -1)                     # noqa: E731
        # both halves leave their heads, times their factor, in one row: [left | right]
        y = ops.new_empty(T, p[pre + "o"].shape[1], dtype=self.dtype, device=self.device)
        H, G, Dv = sp["heads"], sp["kv_heads"], sp["vdim"]
        nl = H * Dv
        kc, vc = cache
        cs = self._rope(pre + "inv_freq", fb, meta, sp["rot_dims"], sp["rot_base"], str(sp["rot_scaling"]))
        qp = ops.qk_norm_rope_kv(part(0, H), part(1, G), part(2, G), None, None, eps, fb.positions, p[pre + "inv_freq"],
                                 fb.slots, kc, vc, cs=cs)
        ops.attn_window_paged(qp, kc, vc, meta["tables"], meta["row_cu"], fb.positions, sp["scale"],
                              min(sp["window"], NO_WINDOW), 0, None, row_map=meta["row_map"], gate=z[:, cut[3]:cut[4]],
                              out_mul=sp["left_scale"], dv_out=Dv, out=y[:, :nl])
        h2 = sp["r_heads"]
        cs = self._rope(pre + "r_inv_freq", fb, meta, sp["r_rot_dims"], sp["r_rot_base"], str(sp["r_rot_scaling"]))
        o = ops.decay_scan(part(4, h2), part(5, h2), part(6, h2), p[pre + "decay"], self.state[sp["index"]],
                           meta["state_slots"], meta["row_cu"], fb.positions, "none", meta["one_row"],
                           p[pre + "r_inv_freq"], cs, sp["r_dim"] ** -0.5)
        ops.head_norm_gate(o, None, eps, z[:, cut[7]:cut[8]], sp["right_scale"], y[:, nl:])
        return self._out(y, p[pre + "o"])

    def _hgrn(self, sp, pre, h, fb, meta):
        T, p, heads = fb.num_tokens, self.p, sp["r_heads"]
        z = ops.linear_act(h, p[pre + "in"])
        n, m = heads * sp["r_dim"], heads * sp["r_vdim"]
        part = lambda a, b: z[:, a:b].view(T, heads, -1)                                       # noqa: E731
        o = ops.forget_scan(part(0, n), part(n, 2 * n), part(2 * n, 2 * n + m), p[pre + "f.b"], p[pre + "lower"],
                            self.state[sp["index"]], meta["state_slots"], meta["row_cu"], fb.positions, "silu",
                            meta["one_row"])
        y = ops.new_empty(T, m, dtype=self.dtype, device=self.device)
        ops.head_norm_gate(o, p[pre + "norm"], self.cfg.norm_eps, None, 1.0, y)
        return self._out(y, p[pre + "o"])

    def _ffn(self, fs, pre, h):
        p = self.p
        if fs["kind"] == "dense":
            return self._glu(pre, h, fs["ff"], NO_LIMIT, RELU, 0.0).contiguous()
        sh = fs["shared"]
        add = self._glu(pre + "shared.", h, sh["ff"], NO_LIMIT, SILU, 0.0) if sh else None
        ids, w = ops.moe_route_scores(h, p[pre + "router"], fs["top"], scoring="softmax", renorm=True,
                                      select_bias=p[pre + "correction"], groups=fs["groups"], renorm_eps=RENORM_EPS,
                                      scale=fs["scale"])
        return ops.moe_glu_ffn(h, ids, w, p[pre + "experts.gate_up"], p[pre + "experts.down"], NO_LIMIT, SILU,
                               up_offset=0.0, scale_input=False, addend=add, identity=fs["identity"] > 0)
