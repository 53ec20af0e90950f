"""Differential attention over the paged cache: two attentions of a head over the same values, and their difference.

Every head has two maps, each with a query and a key of its own (``dim`` features each, projected side by side: head by
head ``[map 1, map 2]``); the values, of a width of their own, are one for both. Query head ``h`` reads kv head
``h // group``. The three projections in carry biases, added before anything else; of each map's first features
neighbouring pairs turn with the position. A row sees the keys up to its own position, or the last ``window`` of them;
each map's weights are an ordinary softmax of ``scale * (q . k)``. With the maps' outputs ``a1`` and ``a2``, per head,

    c = e^(lq1 . lk1) - e^(lq2 . lk2) + diff,      d = a1 - c a2,      out = (1 - diff) d / rms(d)

(``c`` is the layer's, from four learned vectors as long as a map's key; ``rms`` with ``eps`` under the root), and an output
projection without a bias.

A key is cached as one row that holds both maps, so a page serves both with one read and the values are kept once. In
bfloat16 the matrix-core kernels take pages of one width for keys and values, a multiple of 16: the wider of twice a
map's keys (a map's width rounded up to 8) and of the values, with zeros behind what is narrower; with values twice as
wide as a map's keys nothing is padded. Prompts: a wave's two units are a head's two maps, and the difference and its
norm are formed in its registers. Decoding: the maps of all heads of a kv head are rows of one tile, each query in the
half of the row where its keys are, and the kernel that merges the splits of a sequence's keys forms the difference.
Sizes beyond that, and float32, take the kernel of one (row, map) a workgroup and a launch for the difference.
"""

from __future__ import annotations

import math

import torch

from ..cache.spec import KVNeed
from ..cache.store import KVLine
from ..csrc import ops
from ..limits import MATRIX_CORE_HEAD_STEP, MAX_HEAD_DIM
from ..weights.spec import VECTOR
from . import register_part
from .attention import key_splits, keys_seen
from .base import Mixer, Partials, StepContext, matrix
from .linear import linear
from .rope import PairRotaryPositions

_PARTIAL_ROWS = 256         # steps of up to so many rows take the projection as partial sums over K


class DifferentialAttention(Mixer):
    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int, scale: float,
                 diff: float, norm_eps: float, positions: str | None = None, window: int | None = None):
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} query heads cannot share {num_kv_heads} kv heads evenly")
        for name, d in (("head_dim", head_dim), ("value_dim", value_dim)):
            if not 0 < d <= MAX_HEAD_DIM:
                raise ValueError(f"{name} must lie in 1..{MAX_HEAD_DIM}, got {d}")
        self.hidden, self.n_heads, self.n_kv = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.head_dim, self.value_dim = int(head_dim), int(value_dim)
        self.scale, self.diff, self.norm_eps = float(scale), float(diff), float(norm_eps)
        self.positions, self.window = positions, int(window) if window else None
        self.q_dim, self.k_dim = 2 * self.n_heads * self.head_dim, 2 * self.n_kv * self.head_dim
        self.v_dim, self.o_dim = self.n_kv * self.value_dim, self.n_heads * self.value_dim
        self.w_qkv = self.w_o = self.in_bias = None
        self.lam = 0.0

    def tensor_specs(self):
        return {"q_proj": matrix((self.q_dim, self.hidden)), "k_proj": matrix((self.k_dim, self.hidden)),
                "v_proj": matrix((self.v_dim, self.hidden)), "o_proj": matrix((self.hidden, self.o_dim)),
                "q_bias": ((self.q_dim,), VECTOR, "normal"), "k_bias": ((self.k_dim,), VECTOR, "normal"),
                "v_bias": ((self.v_dim,), VECTOR, "normal"),
                **{n: ((self.head_dim,), VECTOR, "normal") for n in ("lq1", "lk1", "lq2", "lk2")}}

    def load(self, tensors):
        self.w_qkv = torch.cat([tensors[n] for n in ("q_proj", "k_proj", "v_proj")], dim=0).contiguous()
        self.w_o = tensors["o_proj"]
        self.in_bias = torch.cat([tensors[n].float() for n in ("q_bias", "k_bias", "v_bias")]).contiguous()
        first, second = (math.exp(float((tensors["lq" + i].double() * tensors["lk" + i].double()).sum())) for i in "12")
        self.lam = first - second + self.diff

    def map_width(self) -> int:
        """Where the second map's keys start in a key's row."""
        return -(-self.head_dim // 8) * 8 if self.page_dim() else self.head_dim

    def page_dim(self) -> int:
        """The one width of keys' and values' pages for the matrix-core kernels (0: those do not serve)."""
        if self.compute_dtype != torch.bfloat16:
            return 0
        wide = max(2 * (-(-self.head_dim // 8) * 8), self.value_dim)
        wide = -(-wide // MATRIX_CORE_HEAD_STEP) * MATRIX_CORE_HEAD_STEP
        return wide if wide <= MAX_HEAD_DIM else 0

    def cache_need(self):
        wide = self.page_dim()
        if wide:
            return KVNeed(self.n_kv, wide, self.window)
        return KVNeed(self.n_kv, 2 * self.head_dim, self.window, self.value_dim if self.value_dim != 2 * self.head_dim else None)

    def kernel_modules(self, dtype):
        return ("gemm", "rope_kv", "attn_rows") + (("attn_mfma",) if dtype == torch.bfloat16 else ())

    def forward(self, h: torch.Tensor, ctx: StepContext, line: KVLine, writes_cache: bool):
        rows, H, G, D, Dv = h.shape[0], self.n_heads, self.n_kv, self.head_dim, self.value_dim
        cos = sin = None
        rot = 0
        if self.positions:
            table = ctx.positions[self.positions]
            if not isinstance(table, PairRotaryPositions):
                raise NotImplementedError("differential attention turns neighbouring pairs (a pair_rotary position encoding)")
            if ctx.max_kv_len > table.n_positions:
                raise ValueError(f"position tables cover {table.n_positions} positions, the step reaches {ctx.max_kv_len}")
            cos, sin, rot = table.cos, table.sin, table.dims
            if rot > D:
                raise ValueError(f"the position encoding rotates {rot} features, a map has {D}")
        proj = linear(h, self.w_qkv, allow_partials=True, partial_rows=_PARTIAL_ROWS)
        if isinstance(proj, Partials):
            proj = (proj.data, proj.count)
        wide, step = self.page_dim(), self.map_width()
        decoding = bool(wide) and ctx.max_q_len == 1
        q = torch.empty((rows, H, 2, wide if decoding else step), dtype=h.dtype, device=h.device)
        ops.rope_maps_kv(proj, 0, self.q_dim, self.q_dim + self.k_dim, self.in_bias, cos, sin, rot, ctx.row_slot, ctx.row_pos, q,
                         step if decoding else 0, line.k, step, line.v, line.page_table, writes_cache, H, G, D, Dv)
        window = self.window or 0
        post = 1.0 - self.diff
        # the tiled prompt kernel never visits the rows of sequences that sit out; they must hold something finite
        out = ctx.kept_zeros((rows, H, Dv), h.dtype) if wide and not decoding and ctx.some_sit_out() else \
            torch.empty((rows, H, Dv), dtype=h.dtype, device=h.device)
        if decoding:
            splits = key_splits(ctx.n_seqs, G * ((2 * H // G + 15) // 16), self.window or ctx.max_kv_len)
            part_o = torch.empty((ctx.n_seqs, 2 * H, splits, wide), dtype=torch.float32, device=h.device)
            part_ml = torch.empty((ctx.n_seqs, 2 * H, splits, 2), dtype=torch.float32, device=h.device)
            ops.attn_split_diff_bf16(q, line.k, line.v, line.page_table, ctx.seq_slot, ctx.cu_rows, ctx.kv_len, ctx.n_seqs,
                                     part_o, part_ml, splits, out, H, G, step, Dv, self.scale, window, self.lam, post,
                                     self.norm_eps)
        elif wide:
            tile_cu, max_tiles = ctx.tiles(ops.ATTN_ROW_TILE)
            ops.attn_causal_diff_bf16(q, line.k, line.v, line.page_table, ctx.seq_slot, ctx.cu_rows, tile_cu, ctx.seq_start,
                                      ctx.n_seqs, max_tiles, out, H, G, step, Dv, self.scale, window, self.lam, post,
                                      self.norm_eps)
        else:
            maps = torch.empty((rows, H, 2, Dv), dtype=h.dtype, device=h.device)
            ops.attn_rows(q, line.k, line.v, line.page_table, ctx.row_slot, ctx.row_pos, maps, 2 * H, G, D, self.scale, window,
                          v_dim=Dv, exact_p=True, maps=2)
            ops.map_difference(maps, out, Dv, self.lam, post, self.norm_eps)
        return linear(out.view(rows, self.o_dim), self.w_o, allow_partials=True)

    def flops(self, rows, spans):
        """The projections, and both products of both maps over the keys each row sees."""
        return super().flops(rows, spans) + 4.0 * self.n_heads * (self.head_dim + self.value_dim) * keys_seen(spans, self.window)


register_part("differential_attention", DifferentialAttention)
