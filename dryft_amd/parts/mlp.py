"""SwiGLU feed-forward: ``down( silu(gate(h)) * up(h) )``, dense, no bias.

Reference: engine/dryft_qwen3/model.py:44-46, 180. Gate and up are fused into one
product by stacking their rows (weights.py:98-100).
"""

from __future__ import annotations

import torch

from ..csrc import ops
from ..weights.spec import VECTOR
from . import register_part
from .base import FeedForward, Partials, matrix
from .linear import STREAM_ROWS, few_rows_ok, linear, panel_swiglu_ok, tall_swiglu_ok


class SwiGLU(FeedForward):
    relu = False              # relu in the place of silu (``ReGLU``)

    def __init__(self, hidden_size: int, intermediate_size: int):
        self.hidden, self.inter = int(hidden_size), int(intermediate_size)
        self.w_gate_up: torch.Tensor | None = None
        self.w_down: torch.Tensor | None = None

    def tensor_specs(self):
        return {"gate_proj": matrix((self.inter, self.hidden)), "up_proj": matrix((self.inter, self.hidden)),
                "down_proj": matrix((self.hidden, self.inter))}

    def load(self, tensors):
        self.w_gate_up = torch.cat([tensors["gate_proj"], tensors["up_proj"]], dim=0).contiguous()
        self.w_down = tensors["down_proj"]

    def kernel_modules(self, dtype):
        return ("gemm", "activation")

    def forward(self, h, ctx):
        act = torch.empty((h.shape[0], self.inter), dtype=h.dtype, device=h.device)
        if h.dtype == torch.bfloat16 and panel_swiglu_ok(h, self.w_gate_up):
            ops.gemm_panel_swiglu_bf16(h, self.w_gate_up, act, relu=self.relu)        # product and activation in one kernel
        elif h.dtype == torch.bfloat16 and tall_swiglu_ok(h, self.w_gate_up):
            ops.gemm_tall_swiglu_bf16(h, self.w_gate_up, act, relu=self.relu)         # the same at 65 to 256 rows
        elif self.relu:
            ops.relu_mul(linear(h, self.w_gate_up), act)
        elif h.dtype == torch.bfloat16 and h.shape[0] <= STREAM_ROWS and few_rows_ok(h, self.w_gate_up):
            ops.gemm_stream_swiglu_bf16(h, self.w_gate_up, act)       # the same for any K that is a multiple of 8
        else:
            ops.silu_mul(linear(h, self.w_gate_up), act)
        return linear(act, self.w_down, allow_partials=True)


class ReGLU(SwiGLU):
    """``down( relu(gate(h)) * up(h) )``, dense, no bias."""

    relu = True


class ClampedGLU(FeedForward):
    """``down( g * sigmoid(alpha * g) * (u + 1) )`` with ``g = min(gate(h), limit)`` and
    ``u = clamp(up(h), -limit, limit)``, dense, no bias. Gate and up are one product, as above."""

    def __init__(self, hidden_size: int, intermediate_size: int, limit: float, alpha: float = 1.702):
        self.hidden, self.inter = int(hidden_size), int(intermediate_size)
        self.limit, self.alpha = float(limit), float(alpha)
        self.w_gate_up: torch.Tensor | None = None
        self.w_down: torch.Tensor | None = None

    def tensor_specs(self):
        return {"gate_proj": matrix((self.inter, self.hidden)), "up_proj": matrix((self.inter, self.hidden)),
                "down_proj": matrix((self.hidden, self.inter))}

    def load(self, tensors):
        self.w_gate_up = torch.cat([tensors["gate_proj"], tensors["up_proj"]], dim=0).contiguous()
        self.w_down = tensors["down_proj"]

    def kernel_modules(self, dtype):
        return ("gemm", "activation")

    def forward(self, h, ctx):
        act = torch.empty((h.shape[0], self.inter), dtype=h.dtype, device=h.device)
        if h.dtype == torch.bfloat16 and panel_swiglu_ok(h, self.w_gate_up):
            # up to 64 rows: product and unit in one kernel, the unit on the float accumulators
            ops.gemm_panel_swiglu_bf16(h, self.w_gate_up, act, clamped=(self.limit, self.alpha))
        else:
            ops.glu_clamped(linear(h, self.w_gate_up), act, self.limit, self.alpha)
        return linear(act, self.w_down, allow_partials=True)


class SquaredReLU(FeedForward):
    """``down( relu(up(h))^2 )``, dense, no gate, no bias."""

    def __init__(self, hidden_size: int, intermediate_size: int):
        self.hidden, self.inter = int(hidden_size), int(intermediate_size)
        self.w_up: torch.Tensor | None = None
        self.w_down: torch.Tensor | None = None

    def tensor_specs(self):
        return {"up_proj": matrix((self.inter, self.hidden)), "down_proj": matrix((self.hidden, self.inter))}

    def load(self, tensors):
        self.w_up, self.w_down = tensors["up_proj"], tensors["down_proj"]

    def kernel_modules(self, dtype):
        return ("gemm", "activation")

    def forward(self, h, ctx):
        act = torch.empty((h.shape[0], self.inter), dtype=h.dtype, device=h.device)
        ops.relu_squared(linear(h, self.w_up), act)
        return linear(act, self.w_down, allow_partials=True)


class PolyNormMLP(FeedForward):
    """``down( c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3 )`` with ``z = up(h)``, powers element by element and ``N`` the division
    of a token's vector by its root mean square (``eps`` inside the root); dense, no bias. Tensor ``act`` holds the four
    numbers. ``z`` reaches the polynomial as the float partial sums of its product where that is split over K."""

    def __init__(self, hidden_size: int, intermediate_size: int, eps: float):
        self.hidden, self.inter, self.eps = int(hidden_size), int(intermediate_size), float(eps)
        self.w_up = self.w_down = self.act = None

    def tensor_specs(self):
        return {"up_proj": matrix((self.inter, self.hidden)), "down_proj": matrix((self.hidden, self.inter)),
                "act": ((4,), VECTOR, "ones")}

    def load(self, tensors):
        self.w_up, self.w_down = tensors["up_proj"], tensors["down_proj"]
        self.act = tensors["act"].float().contiguous()

    def kernel_modules(self, dtype):
        return ("gemm", "activation")

    def forward(self, h, ctx):
        z = linear(h, self.w_up, allow_partials=True)
        act = torch.empty((h.shape[0], self.inter), dtype=h.dtype, device=h.device)
        ops.poly_norm((z.data, z.count) if isinstance(z, Partials) else z, self.act, self.eps, act)
        return linear(act, self.w_down, allow_partials=True)


register_part("swiglu", SwiGLU)
register_part("reglu", ReGLU)
register_part("poly_norm_mlp", PolyNormMLP)
register_part("squared_relu", SquaredReLU)
register_part("clamped_glu", ClampedGLU)
