"""A recurrent mixer whose matrix memory a head is corrected by what it already answers: the gated delta rule, with a
decay a head and key channel.

    [a1 | g1 | q | k | v | b] = W h                     one stacked product
    [z | gate] = [a1 W_a2^T | g1 W_g2^T]                one product of two "heads"
    q, k, v = silu(short causal convolution)            a channel each, `conv_taps` taps
    q, k unit vectors a head (q times q_scale);  f = exp(-exp(a_log) softplus(z + dt_bias));  beta = sigmoid(b)
    S = diag(f) S;  u = beta (v - S^T k);  S = S + k u^T;  o = S^T q      per head, S float32
    out = W_o (o / rms_per_head(o) * w * sigmoid(gate))

Queries and keys may have fewer heads than the values: head h uses q and k head h // (num_heads // num_kv_heads).
The two inner projections (a1, g1) are padded to one size with zero rows, so that the two outer ones are one launch.

A request carries S and the convolutions' last taps - 1 inputs from step to step in one float32 state row of the
cache manager (`ops.delta_state_size` floats, a value column after the other, then [taps - 1, channels]; zeroed at
admission, which is both the zero memory and the zeros before a sequence's start).  The kernels walk every segment's
tokens in order from that row and leave it for the next step, so a prompt may be cut anywhere, and a decoded token
is a segment of one.  Two kernels do so: token by token, or, for the portions of a step that are long enough, chunk by
chunk of 16 tokens on the matrix cores (the same numbers up to the order of float32 sums).  Everything the kernels read of the step lies in device arrays, so a decode step can be
captured in a graph.
"""
from __future__ import annotations

from typing import Optional

import torch

from wllm_amd.kernels import ops
from wllm_amd.parts.common import Product, load_matrix
from wllm_amd.parts.registry import register_mixer
from wllm_amd.parts.specs import DeltaRuleSpec
from wllm_amd.weights.checkpoint import ExpectedTensor, WeightError


# tokens of a request in a step from which its recurrence is walked in chunks (a walk token by token takes 0.17 us a token,
# one in chunks 0.07 and two launches more)
LONG_PORTION = 128


@register_mixer("delta_rule")
class DeltaRuleMixer:
    graph_capturable = True

    def __init__(self, spec: DeltaRuleSpec):
        for name in ("hidden_size", "num_heads", "num_kv_heads", "head_dim", "value_dim", "conv_taps", "decay_rank", "gate_rank"):
            if getattr(spec, name) <= 0:
                raise ValueError(f"{name} must be positive, got {getattr(spec, name)}")
        if spec.num_heads % spec.num_kv_heads:
            raise ValueError(f"num_heads ({spec.num_heads}) must be a multiple of num_kv_heads ({spec.num_kv_heads})")
        if spec.head_dim > ops.DELTA_MAX_DIM:
            raise ValueError(f"head_dim {spec.head_dim}: the recurrence's kernel takes heads of up to {ops.DELTA_MAX_DIM} channels")
        if spec.conv_taps > 64:
            raise ValueError(f"conv_taps {spec.conv_taps}: at most 64")
        self.spec = spec
        self.qk_width = spec.num_kv_heads * spec.head_dim
        self.v_width = spec.num_heads * spec.value_dim
        self.f_width = spec.num_heads * spec.head_dim
        self.channels = 2 * self.qk_width + self.v_width            # what the convolutions run over
        self.outer = max(self.f_width, self.v_width)                # columns of each outer product
        self.memory_size = ops.delta_state_size(spec.num_heads, spec.head_dim, spec.value_dim)
        self._set_inner(max(spec.decay_rank, spec.gate_rank))
        self.w_in = self.t_in = self.w_outer = self.w_o = self.t_o = None
        self.conv_w = self.rate = self.dt_bias = self.norm_w = None

    def _set_inner(self, largest: int) -> None:
        """The inner projections' common size, and where the row's bands then lie."""
        self.inner = -(-largest // 8) * 8
        self.x_offset = 2 * self.inner
        self.b_offset = self.x_offset + self.channels
        self.in_width = -(-(self.b_offset + self.spec.num_heads) // 8) * 8

    def expected_tensors(self) -> dict:
        s = self.spec
        vector, of_norm = dict(role="vector"), dict(role="vector", init="norm")
        return {
            s.q_weight: ExpectedTensor((self.qk_width, s.hidden_size)),
            s.k_weight: ExpectedTensor((self.qk_width, s.hidden_size)),
            s.v_weight: ExpectedTensor((self.v_width, s.hidden_size)),
            s.q_conv_weight: ExpectedTensor((self.qk_width, s.conv_taps), **of_norm),
            s.k_conv_weight: ExpectedTensor((self.qk_width, s.conv_taps), **of_norm),
            s.v_conv_weight: ExpectedTensor((self.v_width, s.conv_taps), **of_norm),
            s.b_weight: ExpectedTensor((s.num_heads, s.hidden_size)),
            s.a1_weight: ExpectedTensor((s.decay_rank, s.hidden_size), free_axes=(0,)),
            s.a2_weight: ExpectedTensor((self.f_width, s.decay_rank), free_axes=(1,)),
            s.a_log: ExpectedTensor((s.num_heads,), **of_norm),
            s.dt_bias: ExpectedTensor((self.f_width,), **of_norm),
            s.g1_weight: ExpectedTensor((s.gate_rank, s.hidden_size), free_axes=(0,)),
            s.g2_weight: ExpectedTensor((self.v_width, s.gate_rank), free_axes=(1,)),
            s.norm_weight: ExpectedTensor((s.value_dim,), **of_norm),
            s.o_weight: ExpectedTensor((s.hidden_size, self.v_width)),
        }

    def load(self, fetch) -> None:
        s = self.spec

        def padded(t: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
            out = torch.zeros(rows, cols, dtype=t.dtype, device=t.device)
            out[:t.shape[0], :t.shape[1]] = t
            return out

        a1, a2, g1, g2 = (fetch.matrix(name) for name in (s.a1_weight, s.a2_weight, s.g1_weight, s.g2_weight))
        for inner, outer, name in ((a1, a2, s.a2_weight), (g1, g2, s.g2_weight)):
            if outer.shape[1] != inner.shape[0]:
                raise WeightError(f"{name}: {outer.shape[1]} columns over an inner projection of {inner.shape[0]} rows",
                                  wrong_shape=[(name, tuple(outer.shape), (outer.shape[0], inner.shape[0]))])
        self._set_inner(max(a1.shape[0], g1.shape[0]))
        w = torch.cat([padded(a1, self.inner, s.hidden_size), padded(g1, self.inner, s.hidden_size)]
                      + [fetch.matrix(name) for name in (s.q_weight, s.k_weight, s.v_weight, s.b_weight)], dim=0)
        self.w_in, self.t_in = load_matrix(fetch, padded(w, self.in_width, s.hidden_size))
        self.w_outer = fetch.to_device(torch.stack([padded(a2, self.outer, self.inner), padded(g2, self.outer, self.inner)]))
        self.w_o, self.t_o = load_matrix(fetch, fetch.matrix(s.o_weight))
        # everything that enters the recurrence, and the convolutions' taps, is kept in float32
        conv = torch.cat([fetch.vector(name) for name in (s.q_conv_weight, s.k_conv_weight, s.v_conv_weight)], dim=0)
        self.conv_w = fetch.to_device(conv.t().contiguous())        # a row a tap
        self.rate = fetch.to_device(torch.exp(fetch.vector(s.a_log)))
        self.dt_bias = fetch.to_device(fetch.vector(s.dt_bias))
        self.norm_w = fetch.to_device(fetch.vector(s.norm_weight).repeat(s.num_heads))

    def cache_need(self):
        return None

    def state_shape(self):
        # (rounded up so that every request's row begins at a multiple of 16 bytes)
        return (-(-(self.memory_size + (self.spec.conv_taps - 1) * self.channels) // 4) * 4,)

    def flops(self, tokens: int, keys: float = 0.0) -> float:
        s = self.spec
        return 2.0 * tokens * (s.hidden_size * (self.in_width + self.v_width) + 2 * self.outer * self.inner
                               + self.channels * s.conv_taps + 4 * self.memory_size)

    def forward(self, ctx, entry: int, h: torch.Tensor, product_input: Optional[torch.Tensor] = None):
        s = self.spec
        n, f32 = h.shape[0], torch.float32
        row = ctx.buffer("delta_in", (n, self.in_width), h.dtype)
        ops.linear(h, self.w_in, row, self.t_in)
        outer = ctx.buffer("delta_outer", (n, 2 * self.outer), h.dtype)
        ops.head_linear(row[:, :2 * self.inner], self.w_outer, outer)
        state = ctx.state(entry)
        dp = ops.delta_padded(s.head_dim)
        qk = ctx.buffer("delta_qk", (2, n, s.num_kv_heads * dp), f32)
        kq = ctx.buffer("delta_kq", (n, s.num_kv_heads), f32)
        f = ctx.buffer("delta_f", (n, s.num_heads * dp), f32)
        beta = ctx.buffer("delta_beta", (n, s.num_heads), f32)
        v = ctx.buffer("delta_v", (n, self.v_width), h.dtype)
        segments = (ctx.seg_q_start, ctx.seg_q_len, ctx.state_slots)
        sizes = dict(heads=s.num_heads, groups=s.num_kv_heads, head_dim=s.head_dim, value_dim=s.value_dim)
        ops.delta_inputs(row[:, self.x_offset:self.b_offset], outer[:, :self.f_width],
                         row[:, self.b_offset:self.b_offset + s.num_heads], self.conv_w, self.rate, self.dt_bias, state,
                         self.memory_size, ctx.token_segment, *segments, qk, kq, v, f, beta, q_scale=s.q_scale,
                         unit_eps=s.unit_eps, single_tokens=ctx.max_q_len == 1 and ctx.num_segments == n, **sizes)
        y = ctx.buffer("delta_y", (n, self.v_width), f32)
        # long portions go 16 tokens at a time over the matrix cores, the others (decoded tokens) token by token
        long = ctx.max_q_len >= LONG_PORTION
        if long:
            chunks = ctx.buffer("delta_chunks", (ops.delta_chunk_size(n, ctx.num_segments, s.num_heads, s.head_dim),), f32)
            ops.delta_chunk_scan(qk, f, beta, v, state, ctx.token_segment, *segments, y, chunks, from_tokens=LONG_PORTION, **sizes)
        if not long or int(ctx.host_q_len.min()) < LONG_PORTION:
            ops.delta_scan(qk, kq, f, beta, v, state, *segments, y, shorter_than=LONG_PORTION if long else None, **sizes)
        out = product_input if product_input is not None else ctx.buffer("delta_out", (n, self.v_width), h.dtype)
        ops.head_norm_gate(y, outer[:, self.outer:self.outer + self.v_width], self.norm_w, out, heads=s.num_heads,
                           eps=s.norm_eps, activation="sigmoid")
        return Product("mixer_out", out, self.w_o, self.t_o)
