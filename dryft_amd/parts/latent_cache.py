"""Attention whose cache holds the latents themselves.

The design of ``LatentAttention`` (queries through a normed latent ``c_q``; plain keys ``U_k c`` and values ``U_v c`` of
every head from a second normed latent ``c``; one rotated key part that all heads share), causal over all earlier
tokens, without sink, window or gate. With nothing to bound what a sequence holds, a token keeps ``kv_rank + rot_dim``
numbers instead of every head's key and value, and a layer may keep nothing and read the line of an earlier layer
(``own_latent=False``: no ``kv_down``, no ``kv_norm``; its run names that layer's cache line and does not write it), with
its own queries, ``U_k`` and ``U_v``.

Two ways of computing the same attention:

* on the latents: a head's query goes to the latent's side, ``U_k^T q_plain``, every head attends to the same cached
  rows, and the weighted sum of latents comes back through ``U_v``. Decoding reads each cached row once for all heads.
  Serves every step.
* with keys and values: for prompts of many rows in bfloat16 that start at a sequence's first token, where every
  (row, earlier row) pair costs ``kv_rank`` operations a head on the latents but only ``dim + rot_dim`` with keys. The
  keys and values of the step's rows are formed once, into pages that live as long as the step, and the prompt kernels
  of the other attention parts serve them.

Float arithmetic in both precisions: both latent norms, the rotation with float32 tables, scores and softmax.
"""

from __future__ import annotations

import numpy as np
import torch

from ..cache.spec import KVNeed, PAGE_TOKENS, pages_for
from ..csrc import ops
from ..limits import MATRIX_CORE_HEAD_STEP, MAX_HEAD_DIM
from ..weights.spec import VECTOR
from . import register_part
from .base import Mixer, Partials, StepContext, matrix
from .linear import linear
from .rope import PairRotaryPositions

_EXPANDED_FROM = 512           # prompts' steps of more rows than this form keys and values (captured steps have fewer)
_WORKGROUPS = 512              # of the kernel that attends to latents: about how many a step is cut into at most


def _padded(w: torch.Tensor, rows_to: int, cols_to: int) -> torch.Tensor:
    """``[heads, n, k]`` with zeros up to multiples of the given numbers of rows and columns."""
    h, n, k = w.shape
    out = torch.zeros((h, -(-n // rows_to) * rows_to, -(-k // cols_to) * cols_to), dtype=w.dtype, device=w.device)
    out[:, :n, :k] = w
    return out


class CachedLatentAttention(Mixer):
    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int, q_rank: int,
                 kv_rank: int, scale: float, norm_eps: float, positions: str | None = None, own_latent: bool = True,
                 name: str = "latent"):
        """``name``: what the layers that read one line are called together (the layer that writes it leaves the
        latents of a step's rows under it for the others)."""
        self.hidden, self.n_heads = int(hidden_size), int(num_heads)
        self.plain, self.rot_dim, self.value_dim = int(head_dim), int(rot_dim), int(value_dim)
        self.key_dim = self.plain + self.rot_dim
        self.q_rank, self.kv_rank = int(q_rank), int(kv_rank)
        self.width = -(-(self.kv_rank + self.rot_dim) // 32) * 32          # of a cached row
        if self.width > ops.LATENT_MAX_WIDTH:
            raise ValueError(f"kv_rank + rot_dim may be at most {ops.LATENT_MAX_WIDTH}, got {kv_rank} + {rot_dim}")
        self.scale, self.norm_eps = float(scale), float(norm_eps)
        self.positions, self.own_latent, self.name = positions, bool(own_latent), str(name)
        self.w_down = self.w_uq = self.w_absorb = self.w_values = self.w_o = self.q_norm = self.kv_norm = None
        self.for_prompts: tuple = ()       # other forms of the same weights that only prompts read

    def tensor_specs(self):
        H = self.n_heads
        specs = {"q_down": matrix((self.q_rank, self.hidden)), "q_norm": ((self.q_rank,), VECTOR, "ones"),
                 "q_up": matrix((H * self.key_dim, self.q_rank)),
                 "k_up": matrix((H * self.plain, self.kv_rank)), "v_up": matrix((H * self.value_dim, self.kv_rank)),
                 "o_proj": matrix((self.hidden, H * self.value_dim))}
        if self.own_latent:
            specs["kv_down"] = matrix((self.kv_rank + self.rot_dim, self.hidden))
            specs["kv_norm"] = ((self.kv_rank,), VECTOR, "ones")
        return specs

    def load(self, tensors):
        H = self.n_heads
        down = [tensors["q_down"]] + ([tensors["kv_down"]] if self.own_latent else [])
        self.w_down = torch.cat(down, dim=0).contiguous()                  # c_q | c | rotated key part
        self.w_uq, self.w_o = tensors["q_up"], tensors["o_proj"]
        k_up, v_up = tensors["k_up"], tensors["v_up"]
        self.w_absorb = _padded(k_up.view(H, self.plain, self.kv_rank).transpose(1, 2), 16, 32)     # U_k^T of every head
        self.w_values = _padded(v_up.view(H, self.value_dim, self.kv_rank), 16, 32)                 # U_v of every head
        wide = self._page_dim()
        if wide:
            o = self.w_o
            if wide != self.value_dim:                                     # the projection skips what heads are padded with
                o = torch.zeros((self.hidden, H, wide), dtype=o.dtype, device=o.device)
                o[:, :, :self.value_dim] = self.w_o.view(self.hidden, H, self.value_dim)
                o = o.view(self.hidden, H * wide)
            self.for_prompts = (torch.cat([k_up, v_up], dim=0).contiguous(), o)
        self.q_norm = tensors["q_norm"].float().contiguous()
        if self.own_latent:
            self.kv_norm = tensors["kv_norm"].float().contiguous()

    def _page_dim(self) -> int:
        """The one width of keys' and values' pages where prompts form them (0: they never do)."""
        step = MATRIX_CORE_HEAD_STEP
        wide = -(-max(self.key_dim, self.value_dim) // step) * step
        return wide if self.compute_dtype == torch.bfloat16 and wide <= MAX_HEAD_DIM else 0

    def cache_need(self):
        return KVNeed(1, self.width, None, 0)

    def kernel_modules(self, dtype):
        return ("gemm", "mla") + (("latent", "attn_mfma") if dtype == torch.bfloat16 else ())

    def _tables(self, ctx: StepContext):
        if not self.positions:
            return None
        table = ctx.positions[self.positions]
        if ctx.max_kv_len > table.n_positions:
            raise ValueError(f"position tables cover {table.n_positions} positions, the step reaches {ctx.max_kv_len}")
        return table.cos, table.sin, table.dims, isinstance(table, PairRotaryPositions)

    def forward(self, h: torch.Tensor, ctx: StepContext, line, writes_cache: bool):
        rows, H = h.shape[0], self.n_heads
        tables = self._tables(ctx)
        # only steps that the host knows have so many rows, and what their sequences start from is part of the step
        many = h.dtype == torch.bfloat16 and ctx.max_q_len > 1 and rows > _EXPANDED_FROM and ctx.host is not None and \
            not any(start for slot, start in zip(ctx.host.slots, ctx.host.starts) if slot >= 0)
        leaves = many and self.own_latent
        down = linear(h, self.w_down, allow_partials=not leaves)
        c_q = torch.empty((rows, self.q_rank), dtype=h.dtype, device=h.device)
        c_kv = torch.empty((rows, self.kv_rank), dtype=h.dtype, device=h.device) if leaves else None
        ops.latent_rows_in((down.data, down.count) if isinstance(down, Partials) else down, self.q_norm, c_q,
                           self.kv_norm, c_kv, self.rot_dim, tables, self.norm_eps, ctx.row_slot, ctx.row_pos, line.k,
                           line.page_table, writes_cache)
        q_raw = linear(c_q, self.w_uq)
        if leaves:
            ctx.shared["latent:" + self.name] = (c_kv, down, self.q_rank)
        if many and self._page_dim():
            return self._with_keys(q_raw, ctx, tables)
        q = torch.empty((rows, H, self.width), dtype=h.dtype, device=h.device)
        ops.head_product(q_raw, 0, self.key_dim, self.w_absorb, self.plain, self.kv_rank, q, self.rot_dim, tables, ctx.row_pos)
        tile_cu, max_tiles = ctx.tiles(ops.latent_tile_rows(H)) if h.dtype == torch.bfloat16 else (None, 0)
        lat = torch.empty((rows, H, self.kv_rank), dtype=h.dtype, device=h.device)
        ops.latent_attend(q, line.k, line.page_table, ctx.seq_slot, ctx.cu_rows, ctx.q_len, ctx.seq_start, tile_cu, ctx.n_seqs,
                          max_tiles, ctx.row_slot, ctx.row_pos, lat, self.kv_rank, self.scale,
                          self._splits(max_tiles, ctx.max_kv_len))
        out = torch.empty((rows, H, self.value_dim), dtype=h.dtype, device=h.device)
        ops.head_product(lat.view(rows, H * self.kv_rank), 0, self.kv_rank, self.w_values, self.kv_rank, self.value_dim, out)
        return linear(out.view(rows, H * self.value_dim), self.w_o, allow_partials=True)

    def _splits(self, tiles: int, max_kv_len: int) -> int:
        """Into how many runs a sequence's keys are cut: as many as fill the chip, at most one per run of keys that the
        kernel takes at a time, and no more than the runs of equal length that this leaves need."""
        blocks, pieces = max(1, tiles) * -(-self.n_heads // 16), -(-max_kv_len // ops.LATENT_KEYS)
        most = max(1, min(_WORKGROUPS // blocks, ops.LATENT_MAX_SPLITS, pieces))
        return -(-pieces // -(-pieces // most))

    def _with_keys(self, q_raw: torch.Tensor, ctx: StepContext, tables):
        rows, H, dev = q_raw.shape[0], self.n_heads, q_raw.device
        found = ctx.shared.get("latent:" + self.name)
        if found is None or found[0].shape != (rows, self.kv_rank):
            raise ValueError(f"latent {self.name!r}: no earlier layer of this step has left one of this width")
        c_kv, down, lat_col = found                                         # of the layer that writes the line
        table, n_pages = self._step_pages(ctx)
        wide = self._page_dim()
        # zeros once a step: a layer's pages are overwritten by the next one's, finite wherever no row is
        k = ctx.kept_zeros((2, n_pages, H, PAGE_TOKENS, wide), q_raw.dtype)
        k, v = k[0], k[1].view(n_pages, H, wide, PAGE_TOKENS)
        w_ukv, w_o = self.for_prompts
        kv = linear(c_kv, w_ukv)                                            # plain keys of all heads | values of all heads
        q = torch.empty((rows, H, wide), dtype=q_raw.dtype, device=dev)
        cos, sin, rot, pairs = tables if tables is not None else (None, None, 0, False)
        ops.latent_rope_kv(q_raw, kv, down, lat_col + self.kv_rank, cos, sin, rot, ctx.row_slot, ctx.row_pos, q, k, v, table, True, H,
                           self.plain, self.rot_dim, self.value_dim, wide, pairs=pairs, page_dk=wide)
        out = ctx.kept_zeros((rows, H, wide), q_raw.dtype) if ctx.some_sit_out() else \
            torch.empty((rows, H, wide), dtype=q_raw.dtype, device=dev)
        tile_cu, max_tiles = ctx.tiles(ops.ATTN_ROW_TILE)
        ops.attn_causal_bf16(q, k, v, table, ctx.seq_slot, ctx.cu_rows, tile_cu, ctx.seq_start, ctx.n_seqs, max_tiles, out, H, H,
                             wide, self.scale, 0)
        return linear(out.view(rows, H * wide), w_o, allow_partials=True)

    @staticmethod
    def _step_pages(ctx: StepContext):
        """A page table for the step's own keys and values: the live sequences' pages one after another (one table a step)."""
        found = ctx.shared.get("latent:pages")
        if found is None:
            need = [pages_for(q) if s >= 0 else 0 for s, q in zip(ctx.host.slots, ctx.host.q_lens)]
            table = np.full((max(ctx.host.slots) + 1, max(need)), -1, dtype=np.int32)
            at = 0
            for slot, n in zip(ctx.host.slots, need):
                if n:
                    table[slot, :n] = np.arange(at, at + n)
                at += n
            found = ctx.shared["latent:pages"] = (torch.from_numpy(table).to(ctx.device), at)
        return found

    def flops(self, rows, spans):
        seen = sum((2 * start + q + 1) * q // 2 for start, q in spans)
        return super().flops(rows, spans) + 2.0 * self.n_heads * (self.key_dim + self.value_dim) * seen


register_part("cached_latent_attention", CachedLatentAttention)
