"""Feed-forward parts.  "gated_mlp": down(act(gate(x)) * up(x)) without biases;
with act = gelu_tanh it is the reference's GemmaMLP (src/wllm/models/gemma.py:54-62).
"clamped_swish" holds the gate under a limit and the up projection between two, and raises the latter by a constant.
Gate and up matrices are stacked at load so that one product makes both halves
of the row the activation kernel reads.  "mlp": down(act(up(x))), no gate."""
from __future__ import annotations

import torch

from wllm_amd.kernels import ops
from wllm_amd.parts.common import Product, load_matrix
from wllm_amd.parts.registry import register_feed_forward
from wllm_amd.parts.specs import GatedMLPSpec, MLPSpec
from wllm_amd.weights.checkpoint import ExpectedTensor


@register_feed_forward("gated_mlp")
class GatedMLP:
    def __init__(self, spec: GatedMLPSpec):
        if spec.activation == "clamped_swish":
            if spec.gate_limit is None:
                raise ValueError("a clamped swish needs gate_limit")
            self.activation = ops.ClampedSwish(spec.gate_limit, spec.gate_slope, spec.up_shift)
        elif spec.activation in ops.ACTIVATIONS:
            if spec.gate_limit is not None or spec.gate_slope != 1.0 or spec.up_shift != 0.0:
                raise ValueError(f"activation {spec.activation!r} takes no limit, slope or shift")
            self.activation = spec.activation
        else:
            raise ValueError(f"activation {spec.activation!r} is not implemented; known: {ops.ACTIVATIONS} and clamped_swish")
        self.spec = spec
        self.w_gate_up = self.t_gate_up = None      # the matrix and its tile-major copy
        self.w_down = self.t_down = None

    def expected_tensors(self) -> dict:
        s = self.spec
        return {
            s.gate_weight: ExpectedTensor((s.intermediate_size, s.hidden_size)),
            s.up_weight: ExpectedTensor((s.intermediate_size, s.hidden_size)),
            s.down_weight: ExpectedTensor((s.hidden_size, s.intermediate_size)),
        }

    def load(self, fetch) -> None:
        s = self.spec
        self.w_gate_up, self.t_gate_up = load_matrix(
            fetch, torch.cat([fetch.matrix(s.gate_weight), fetch.matrix(s.up_weight)], dim=0), halves=2)
        self.w_down, self.t_down = load_matrix(fetch, fetch.matrix(s.down_weight))

    def flops(self, tokens: int) -> float:
        """Floating-point operations of `tokens` tokens (what a measurement divides by its time)."""
        return 6.0 * tokens * self.spec.hidden_size * self.spec.intermediate_size

    def takes_norm_on_load(self, rows: int, dtype: torch.dtype) -> bool:
        """Whether `forward` may be given `ops.NormOnLoad` instead of the normalised tensor."""
        return ops.gated_linear_norm_takes(rows, dtype, self.spec.hidden_size)

    def forward(self, ctx, h, product_input=None):
        """`product_input`: a band of columns [n, intermediate] of a wider buffer into which the input
        of the down projection is to be written (a block that makes one product of several parts'
        last products asks for it); the returned `Product` then names that band."""
        s = self.spec
        n = h.shape[0]
        if isinstance(h, ops.NormOnLoad):
            act = ctx.buffer("ffn_act", (n, s.intermediate_size), h.dtype)
            ops.gated_linear(h, self.w_gate_up, act, self.activation, None, self.t_gate_up)
        else:
            gate_up = ctx.buffer("gate_up", (n, 2 * s.intermediate_size), h.dtype)
            if (product_input is not None and ops.gated_linear_writes_band(n, h.dtype, s.hidden_size)
                    and product_input.data_ptr() % 16 == 0 and product_input.stride(0) % 8 == 0):
                act = product_input         # the kernel writes the band itself (its rows begin at multiples of 16 bytes)
            else:
                act = ctx.buffer("ffn_act", (n, s.intermediate_size), h.dtype)
            ops.gated_linear(h, self.w_gate_up, act, self.activation, gate_up, self.t_gate_up)
        if product_input is not None and act is not product_input:
            ops.copy_columns(act, product_input)
            act = product_input
        return Product("ffn_out", act, self.w_down, self.t_down)


@register_feed_forward("mlp")
class MLP:
    """down(act(up(x))).  Where the few-row and tiled kernels of a gated product apply (bfloat16, an even number of
    columns), the two halves of the columns are their two streams and the activation is made in their registers."""

    def __init__(self, spec: MLPSpec):
        if spec.activation not in ops.SINGLE_ACTIVATIONS:
            raise ValueError(f"activation {spec.activation!r} is not implemented; known: {sorted(ops.SINGLE_ACTIVATIONS)}")
        self.spec = spec
        self.w_up = self.t_up = self.w_down = self.t_down = None
        self.paired = False                 # t_up is tiled as two halves

    def expected_tensors(self) -> dict:
        s = self.spec
        return {s.up_weight: ExpectedTensor((s.intermediate_size, s.hidden_size)),
                s.down_weight: ExpectedTensor((s.hidden_size, s.intermediate_size))}

    def load(self, fetch) -> None:
        s = self.spec
        self.paired = s.intermediate_size % 2 == 0 and fetch.dtype == torch.bfloat16
        self.w_up, self.t_up = load_matrix(fetch, fetch.matrix(s.up_weight), halves=2 if self.paired else 1)
        self.w_down, self.t_down = load_matrix(fetch, fetch.matrix(s.down_weight))

    def flops(self, tokens: int) -> float:
        return 4.0 * tokens * self.spec.hidden_size * self.spec.intermediate_size

    def forward(self, ctx, h, product_input=None):
        s = self.spec
        act = ctx.buffer("ffn_act", (h.shape[0], s.intermediate_size), h.dtype)
        ops.activated_linear(h, self.w_up, act, s.activation, None if self.paired else self.t_up,
                             self.t_up if self.paired else None)
        if product_input is not None:
            ops.copy_columns(act, product_input)
            act = product_input
        return Product("ffn_out", act, self.w_down, self.t_down)
