"""What the heterogeneous layer stacks (models/nesizen.py, zinesun.py and the others) share: unsharded
single-rank models whose steps are packed rows (decoded rows first, then prompt chunks) that
always attend through the paged cache."""
from __future__ import annotations

from typing import Optional

import torch

from .. import ops
from ..engine.batch import ForwardBatch


def pad128(n: int) -> int:
    """Fused projections carry zero rows up to a multiple of 128 (the MFMA GEMMs' N tiling)."""
    return (n + 127) // 128 * 128


class PackedStack:
    """Mixin: expects self.p (parameter dict), self.cfg, self.device, self.dtype, self.specs,
    self.has_state."""
    paged_prefill_only = True     # the runner builds block tables for every prompt chunk
    supports_f32 = True           # every kernel of the family has a true 32-bit form
    attention_types = ("attention",)

    def local_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.p.values() if t is not None)

    def packed_decode_bytes(self, kinds=None) -> int:
        return 0

    def pack_decode_weights(self, budget_bytes=None, kinds=None) -> int:
        return 0

    def kv_bytes_per_token(self, dtype: Optional[torch.dtype] = None) -> int:
        es = torch.empty((), dtype=dtype or self.dtype).element_size()
        return max(1, self.cfg.kv_bytes_per_token(es))

    def gemm_shapes(self) -> list:
        return sorted({tuple(w.shape) for k, w in self.p.items()
                       if w is not None and w.dim() == 2 and w.dtype == torch.bfloat16 and k != "embed"
                       and w.shape[0] % 128 == 0 and w.shape[1] % 64 == 0})

    def _wide(self, rows: int, k: int) -> int:
        """Rows of a projection: padded to the tuned GEMMs' 128-row tiling when its K fits them."""
        return pad128(rows) if k % 64 == 0 else rows

    # a GLU feed-forward W_down (act(W_gate h) * (W_up h)) without biases: fused [gate | up] rows under
    # self.p[name + "gate_up"], self.p[name + "down"]
    def _glu_group(self, ff: int) -> int:
        """Row group of a GLU's [gate | up] weight: alternating 16-row blocks where the tuned GEMMs can run
        the activation as their epilogue, else 0 (all gate rows, then all up rows)."""
        fused = self.dtype == torch.bfloat16 and self.device.type == "cuda" and self.cfg.hidden_size % 64 == 0 and ff % 128 == 0
        return ops.SILU_INTERLEAVE if fused else 0

    def _glu_alloc(self, name: str, ff: int, limit: float, alpha: float, offset: float) -> None:
        z = lambda *s: torch.zeros(*s, dtype=self.dtype, device=self.device)                  # noqa: E731
        W = self.cfg.hidden_size
        if self._glu_group(ff):
            self.p[name + "gate_up"] = z(2 * ff, W)
            self.p[name + "gate_up.b"] = ops.glu_bias_block(z(2 * ff), limit, alpha, offset)
        else:
            self.p[name + "gate_up"] = z(self._wide(2 * ff, W), W)
        self.p[name + "down"] = z(self._wide(W, ff), ff)

    def _glu_logical(self, add, name: str, local: str, ff: int) -> None:
        """The GLU's checkpoint tensors `name`gate / up / down as views into the fused local tensors."""
        W, w, grp = self.cfg.hidden_size, self.p[local + "gate_up"], self._glu_group(ff)
        if grp:        # alternating blocks of `grp` gate and up rows
            wv = w.view(ff // grp, 2, grp, W)
            for j, n in enumerate(("gate", "up")):
                add(name + n, wv[:, j], shape=(ff, W), get=lambda t=wv[:, j]: t.reshape(-1, t.shape[-1]))
        else:
            add(name + "gate", w[:ff])
            add(name + "up", w[ff:2 * ff])
        add(name + "down", self.p[local + "down"][:W])

    def _glu(self, name: str, h, ff: int, limit: float, alpha: float, offset: float):
        p = self.p
        a = ops.linear_glu(h, p[name + "gate_up"], p.get(name + "gate_up.b"), ff, limit, alpha, offset, self._glu_group(ff))
        return ops.linear_act(a, p[name + "down"])[:, :self.cfg.hidden_size]

    def _iota(self, n: int) -> torch.Tensor:
        t = self._arange.get(n)
        if t is None:
            t = self._arange[n] = torch.arange(n, dtype=torch.int32, device=self.device)
        return t

    def _step_meta(self, fb: ForwardBatch) -> dict:
        """Packed-row description shared by the mixers: row_cu [nseq + 1] (decode rows are
        one-row sequences, then the prompt chunks), one block table per sequence, state slots."""
        T = fb.num_tokens
        name = type(self).__name__
        if not fb.is_prefill:
            row_cu, tables = self._iota(T + 1), fb.block_tables
        else:
            nd = fb.num_decode
            if fb.cu_seqlens.numel() > 1 and fb.prefix_tables is None:
                raise RuntimeError(f"{name}: prompt chunks need their block tables (mixed scheduling)")
            if nd:
                row_cu = torch.cat([self._iota(nd), fb.cu_seqlens + nd])
                tables = fb.block_tables[:nd] if fb.prefix_tables is None else torch.cat([fb.block_tables[:nd], fb.prefix_tables])
            else:
                row_cu, tables = fb.cu_seqlens, fb.prefix_tables
        m = {"row_cu": row_cu, "tables": tables, "state_slots": fb.state_slots, "row_map": None}
        if self.has_state and fb.state_slots is None and T:
            raise RuntimeError(f"{name}: the batch carries no per-sequence state slots")
        if self.device.type == "cuda" and T and any(sp["type"] in self.attention_types for sp in self.specs):
            m["row_map"] = ops.row_seq(row_cu, T)
        return m
