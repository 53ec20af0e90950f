"""Linear attention: a matrix state per head that decays and takes ``k v^T`` of every token, read out by ``q``.

Per head ``S <- diag(alpha_t) S + k_t v_t^T`` and ``o_t = S^T q_t`` with the new state; no softmax, no denominator. ``q``,
``k``, ``v`` and a gate are projections without biases; ``q`` and ``k`` may be turned by a rotation over halves and are
multiplied by ``q_scale`` and ``k_scale``. The decay is one of two kinds:

* ``head_decay``: a fixed number per head (retention);
* ``channel_decay = (rank, tau)``: a number per head, key channel and token, ``sigmoid(W_up (W_down h) + b)^(1 / tau)``
  (gated linear attention; ``rank`` -1: whatever the checkpoint holds).

Each head's ``o`` is divided by its root mean square (``eps`` inside the root), with ``out_norm`` times a weight that all
heads share, times ``silu`` of the gate, and projected back.

The state is float32 in the state store, zero when a sequence starts. The decays keep the float accumulators of their
first projection; they, the rotated ``q`` and ``k``, the recurrence, the read-out and its norm are float arithmetic in
both precisions. Steps of one row a sequence run as one kernel from the projection to the gated read-out; steps that
bring more run sixteen tokens at a time on the matrix cores in 32-bit precision, long sequences as segments side by side.
"""

from __future__ import annotations

import torch

from ..cache.spec import StateNeed
from ..csrc import ops
from ..weights.spec import VECTOR
from . import register_part
from .base import Mixer, StepContext, matrix
from .linear import linear
from .rope import HalfRotaryPositions


class LinearAttention(Mixer):
    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, norm_eps: float,
                 head_decay: list[float] | None = None, channel_decay: tuple[int, float] | None = None,
                 positions: str | None = None, q_scale: float = 1.0, k_scale: float = 1.0, out_norm: bool = False):
        self.hidden, self.n_heads, self.key_dim, self.value_dim = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        if not (0 < self.key_dim <= ops.LINEAR_MAX_DIM and 0 < self.value_dim <= ops.LINEAR_MAX_DIM):
            raise ValueError(f"key_dim and value_dim must lie in 1..{ops.LINEAR_MAX_DIM}, got {key_dim} and {value_dim}")
        if (head_decay is None) == (channel_decay is None):
            raise ValueError("decays are fixed per head (head_decay) or come from the input (channel_decay), one of the two")
        self.head_decay = [float(d) for d in head_decay] if head_decay is not None else None
        if self.head_decay is not None and (len(self.head_decay) != self.n_heads or not all(0 < d <= 1 for d in self.head_decay)):
            raise ValueError(f"head_decay needs a number in (0, 1] for each of {num_heads} heads")
        self.channel_decay = (int(channel_decay[0]), float(channel_decay[1])) if channel_decay is not None else None
        self.norm_eps, self.positions = float(norm_eps), positions
        self.q_scale, self.k_scale, self.has_norm = float(q_scale), float(k_scale), bool(out_norm)
        self.qk_dim, self.v_dim = self.n_heads * self.key_dim, self.n_heads * self.value_dim
        self.w_in = self.w_down = self.w_up = self.decay_bias = self.w_o = self.out_norm = self.out_norm_all = None
        self.decays = self.log_decays = None

    def tensor_specs(self):
        specs = {"q_proj": matrix((self.qk_dim, self.hidden)), "k_proj": matrix((self.qk_dim, self.hidden)),
                 "v_proj": matrix((self.v_dim, self.hidden)), "g_proj": matrix((self.v_dim, self.hidden)),
                 "o_proj": matrix((self.hidden, self.v_dim))}
        if self.channel_decay:
            rank = self.channel_decay[0]
            specs.update({"decay_down": matrix((rank, self.hidden)), "decay_up": matrix((self.qk_dim, rank)),
                          "decay_bias": ((self.qk_dim,), VECTOR, "normal")})
        if self.has_norm:
            specs["out_norm"] = ((self.value_dim,), VECTOR, "ones")
        return specs

    def load(self, tensors):
        self.w_in = torch.cat([tensors[n] for n in ("q_proj", "k_proj", "v_proj", "g_proj")], dim=0).contiguous()
        self.w_o = tensors["o_proj"]
        device = self.w_in.device
        if self.channel_decay:
            self.w_down, self.w_up = tensors["decay_down"], tensors["decay_up"].contiguous()
            if self.w_down.shape[0] != self.w_up.shape[1]:
                raise ValueError(f"the decay's two projections disagree on its rank: {tuple(self.w_down.shape)} and "
                                 f"{tuple(self.w_up.shape)}")
            self.decay_bias = tensors["decay_bias"].float().contiguous()
        else:
            decay = torch.tensor(self.head_decay, dtype=torch.float64)
            self.decays = decay.to(torch.float32).to(device)
            self.log_decays = self.decays.double().log().to(torch.float32).contiguous()
        if self.has_norm:
            self.out_norm = tensors["out_norm"].float().contiguous()
        weight = self.out_norm if self.has_norm else torch.ones(self.value_dim, dtype=torch.float32, device=device)
        self.out_norm_all = weight.repeat(self.n_heads).contiguous()         # head by head, for the kernel after a prompt

    def cache_need(self):
        return StateNeed((self.n_heads, self.key_dim, self.value_dim))

    def kernel_modules(self, dtype):
        return ("gemm", "linattn", "wkv")

    def _tables(self, ctx: StepContext):
        if not self.positions:
            return None
        table = ctx.positions[self.positions]
        if not isinstance(table, HalfRotaryPositions):
            raise NotImplementedError("linear attention turns q and k over halves with float tables")
        if ctx.max_kv_len > table.n_positions:
            raise ValueError(f"position tables cover {table.n_positions} positions, the step reaches {ctx.max_kv_len}")
        return table.cos, table.sin, table.dims

    def forward(self, h: torch.Tensor, ctx: StepContext, line, writes_cache: bool):
        rows = h.shape[0]
        proj = linear(h, self.w_in)                                       # q | k | v | gate
        logs = None
        if self.channel_decay:
            low = linear(h, self.w_down, out_dtype=torch.float32)          # the decay stays float32 from here on
            logs = torch.empty((rows, self.qk_dim), dtype=torch.float32, device=h.device)
            ops.log_decay(low, self.w_up, self.decay_bias, logs, 1.0 / self.channel_decay[1])
        cols = (0, self.qk_dim, 2 * self.qk_dim)
        g_col = 2 * self.qk_dim + self.v_dim
        tables = self._tables(ctx)
        out = torch.empty((rows, self.v_dim), dtype=h.dtype, device=h.device)
        if ctx.max_q_len == 1:
            ops.linear_token(proj, *cols, g_col, self.q_scale, self.k_scale, tables, ctx.row_pos, logs, self.decays,
                             ctx.seq_slot, ctx.cu_rows, ctx.q_len, ctx.n_seqs, line.state, self.out_norm, self.norm_eps, out,
                             self.n_heads, self.key_dim, self.value_dim, writes_cache)
            return linear(out, self.w_o, allow_partials=True)
        # a long prompt runs as segments side by side (the rows of sequences that sit out are then not visited)
        segments = ctx.segments(ops.LINEAR_CHUNK) if writes_cache else None
        if segments is not None and ctx.some_sit_out():
            o_raw = ctx.kept_zeros((rows, self.v_dim), torch.float32)
        else:
            o_raw = torch.empty((rows, self.v_dim), dtype=torch.float32, device=h.device)
        ops.linear_chunks(proj, *cols, self.q_scale, self.k_scale, tables, ctx.row_pos, logs, self.log_decays, ctx.seq_slot,
                          ctx.cu_rows, ctx.q_len, ctx.n_seqs, line.state, o_raw, self.n_heads, self.key_dim, self.value_dim,
                          writes_cache, segments=segments)
        ops.wkv_out(o_raw, proj[:, g_col:], self.out_norm_all, out, self.n_heads, self.value_dim, self.norm_eps)
        return linear(out, self.w_o, allow_partials=True)

    def flops(self, rows, spans):
        """The projections, and per token and head the update of the state and its read-out."""
        return super().flops(rows, spans) + 5.0 * rows * self.n_heads * self.key_dim * self.value_dim


register_part("linear_attention", LinearAttention)
