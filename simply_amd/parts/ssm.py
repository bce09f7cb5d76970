"""A state-space recurrent mixer with one decay per head.  From one projection of the mixer's input, [z | x | B | C | p]:
x (heads x value size), B and C (groups x state size) pass a causal convolution per channel with a bias, then silu; per
head the step size dt = softplus(p + dt_bias).  Head h reads the B and C of group h // (heads / groups), and with its state
S [state size, value size] from zero,

    S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T,      y_t = S_t^T C_t + D x_t

y (heads side by side) is multiplied by silu(z), then normed in equal parts of the channels, each by its own root mean
square, multiplied by a weight per channel and projected.  A request's state is S and the convolution's last taps - 1
inputs, one float32 row of a state slot; step sizes, decays, S and the norm are 32-bit, the projections and the
convolution's result have the activation type."""
from __future__ import annotations

import torch

from ..kernels import ops
from ..registry import MIXERS
from .base import Mixer, ParamSpec, StateNeed, as_product_weight, project


@MIXERS.register("state_space")
class StateSpace(Mixer):
    #: the mixer's input enters one product only: for a few rows the norm in front of it runs in that product's kernel
    accepts_pending = True
    defers_sum = True
    #: tokens of a request in a step from which the recurrence is worked through in pieces
    PIECES_FROM = 12

    def __init__(self, hidden_size: int, num_heads: int, num_groups: int, state_dim: int, value_dim: int, conv_taps: int,
                 norm_groups: int, norm_eps: float):
        self.hidden_size, self.num_heads, self.num_groups = int(hidden_size), int(num_heads), int(num_groups)
        self.state_dim, self.value_dim, self.conv_taps = int(state_dim), int(value_dim), int(conv_taps)
        self.norm_groups, self.norm_eps = int(norm_groups), float(norm_eps)
        if self.num_heads % self.num_groups:
            raise ValueError(f"state_space: {num_heads} heads do not split over {num_groups} groups")
        if self.conv_taps < 1:
            raise ValueError("state_space: the convolution has at least one tap")
        self.inner = self.num_heads * self.value_dim
        if self.inner % self.norm_groups:
            raise ValueError(f"state_space: {self.inner} channels do not split into {norm_groups} equal parts")
        #: channels that pass the convolution: x, then B and C of every group
        self.channels = self.inner + 2 * self.num_groups * self.state_dim
        #: rows of the projection, with rows of zeros behind it so that its results' rows start at aligned addresses
        self.rows = self.inner + self.channels + self.num_heads
        self.padded_rows = -(-self.rows // 8) * 8
        self.state_words = self.num_heads * self.state_dim * self.value_dim
        # (the tails start at a multiple of four words, for 16-byte accesses)
        self.tails_at = -(-self.state_words // 4) * 4
        self.in_proj = self.o_proj = self.taps = self.conv_bias = self.dt_bias = self.a_log = self.skip = self.norm = None

    def param_specs(self):
        D, H, C, n = self.hidden_size, self.num_heads, self.channels, self.conv_taps
        vec = dict(role="vector", init="norm")
        return {"in_proj": ParamSpec((self.rows, D)), "conv": ParamSpec((C, n), role="vector"),
                "conv_bias": ParamSpec((C,), **vec), "dt_bias": ParamSpec((H,), **vec), "a_log": ParamSpec((H,), **vec),
                "skip": ParamSpec((H,), **vec), "norm": ParamSpec((self.inner,), **vec),
                "o_proj": ParamSpec((D, self.inner))}

    def load(self, tensors):
        t = tensors
        w = t["in_proj"]
        if self.padded_rows != self.rows:
            w = torch.cat([w, torch.zeros((self.padded_rows - self.rows, w.shape[1]), dtype=w.dtype, device=w.device)])
        self.in_proj = as_product_weight(w.contiguous())
        self.o_proj = as_product_weight(t["o_proj"])
        self.taps = t["conv"].t().contiguous()   # [taps, channels]
        self.conv_bias = t["conv_bias"].to(self.taps.dtype).contiguous()
        self.dt_bias, self.a_log = t["dt_bias"].contiguous(), t["a_log"].to(t["dt_bias"].dtype).contiguous()
        self.skip, self.norm = t["skip"].contiguous(), t["norm"].contiguous()

    def cache_need(self):
        return StateNeed((self.tails_at + (self.conv_taps - 1) * self.channels,), torch.float32)

    def forward(self, x, ctx, cache, defer_sum=False):
        if not cache.write:
            raise RuntimeError("state_space: a recurrent state cannot be read through another entry's cache")
        H, G, N, dv, inner = self.num_heads, self.num_groups, self.state_dim, self.value_dim, self.inner
        proj = project(x, self.in_proj)
        u, gates = ops.ssm_inputs(proj, inner, inner + self.channels, self.channels, H, self.taps, self.conv_bias,
                                  self.dt_bias, self.a_log, cache.state[:, self.tails_at:], ctx.seq_meta, ctx.num_seqs,
                                  ctx.max_q_len)
        # queries C, keys B, values x; a decay and an input factor (the step size) per head.  Requests with few tokens go
        # through the recurrence token by token, portions of prompts in pieces on the matrix cores where these take the sizes
        at = (inner + G * N, inner, 0)
        y = torch.empty((u.shape[0], inner), dtype=torch.float32, device=u.device)
        short = ctx.num_seqs
        if ctx.max_q_len >= self.PIECES_FROM and ops.state_chunks_takes(u, *at, N, dv, cache.state):
            short, _ = ctx.short_requests(self.PIECES_FROM - 1)
            ops.state_chunks(u, *at, gates, H, G, N, dv, cache.state, ctx.seq_meta[short:], ctx.num_seqs - short,
                             skip=self.skip, out=y)
        if short:
            ops.linear_state(u, *at, 1.0, gates, True, H, N, dv, False, cache.state, ctx.seq_meta, short, key_heads=G,
                             skip=self.skip, out=y)
        z = ops.gated_group_norm(y, proj[:, :inner], self.norm_groups, self.norm, self.norm_eps)
        return ops.gemm(z, self.o_proj, defer_sum=defer_sum)
