"""Time mixing with a token shift, data-dependent decays and a bonus for the current token.

Every one of the five streams r, k, v, g, w reads a mix of the token's input h and the one before it, h' (zeros before a
sequence's first token), h + (h' - h) * mu_s.  r, k, v (heads x size) and the gate are projections of their mixes; the
decay per head and key channel is a = exp(-exp(W_2 tanh(W_1 mix_w) + w_0)).  Per head, with S [size, size] from zero,

    o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,      S_t = diag(a_t) S_(t-1) + k_t v_t^T

and each head's o is divided by its root mean square, multiplied by a weight (one entry per head and channel) and by
silu(gate), then projected.  A request's state is S and its last h, one float32 row of a state slot; mixes, decays, S and
the norm are 32-bit, the projections read and give the activation type."""
from __future__ import annotations

import torch

from ..kernels import ops
from ..registry import MIXERS
from .base import Mixer, ParamSpec, StateNeed, as_product_weight


@MIXERS.register("wkv")
class WKV(Mixer):
    STREAMS = ("r", "k", "v", "g", "w")

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, decay_rank: int, norm_eps: float):
        self.hidden_size, self.num_heads, self.head_dim = int(hidden_size), int(num_heads), int(head_dim)
        self.decay_rank, self.norm_eps = int(decay_rank), float(norm_eps)
        self.state_words = self.num_heads * self.head_dim * self.head_dim
        self.mu = self.in_proj = self.decay_out = self.decay_base = self.bonus = self.norm = self.o_proj = None

    def param_specs(self):
        D, H, d, R = self.hidden_size, self.num_heads, self.head_dim, self.decay_rank
        vec = dict(role="vector", init="norm")
        specs = {"mu_" + s: ParamSpec((D,), **vec) for s in self.STREAMS}
        specs.update({s + "_proj": ParamSpec((H * d, D)) for s in "rkvg"})
        specs.update(decay_in=ParamSpec((R, D)), decay_out=ParamSpec((H * d, R)), decay_base=ParamSpec((H * d,), **vec),
                     bonus=ParamSpec((H, d), **vec), norm=ParamSpec((H * d,), **vec), o_proj=ParamSpec((D, H * d)))
        return specs

    def load(self, tensors):
        t = tensors
        self.mu = torch.stack([t["mu_" + s].to(t["mu_r"].dtype) for s in self.STREAMS]).contiguous()
        # r, k, v, the gate and the decay's first factor: products whose blocks of outputs read blocks of the mixes, run
        # as one where the decay's rank is not larger than the heads
        rkvg = [t[s + "_proj"] for s in "rkvg"]
        self.decay_in = None if self.decay_rank <= rkvg[0].shape[0] else as_product_weight(t["decay_in"])
        self.in_proj = ops.SectionedWeight(rkvg + ([t["decay_in"]] if self.decay_in is None else []))
        self.decay_out = as_product_weight(t["decay_out"])
        self.decay_base, self.norm = t["decay_base"].contiguous(), t["norm"].contiguous()
        self.bonus = t["bonus"].reshape(-1).contiguous()
        self.o_proj = as_product_weight(t["o_proj"])

    def cache_need(self):
        return StateNeed((self.state_words + self.hidden_size,), torch.float32)   # S, then the last token's h

    def forward(self, x, ctx, cache):
        if not cache.write:
            raise RuntimeError("wkv: a recurrent state cannot be read through another entry's cache")
        D, H, d = self.hidden_size, self.num_heads, self.head_dim
        C = H * d
        mixes = ops.token_shift(x, self.mu, cache.state[:, self.state_words:], ctx.seq_meta, ctx.num_seqs, ctx.max_q_len)
        if self.decay_in is None:
            proj = ops.gemm_sections(mixes, self.in_proj)                             # [T, r | k | v | gate | decay's factor]
            low = proj[:, 4 * C:]
        else:
            proj, low = ops.gemm_sections(mixes[:, :4 * D], self.in_proj), ops.gemm(mixes[:, 4 * D:], self.decay_in)
        decay = ops.low_rank_decay(low, self.decay_out, self.decay_base)
        o = ops.linear_state(proj, 0, C, 2 * C, 1.0, decay, False, H, d, d, False, cache.state, ctx.seq_meta, ctx.num_seqs,
                             bonus=self.bonus)
        z = ops.gated_heads(o, proj[:, 3 * C:4 * C], H, d, kind=ops.GATE_SILU, weight=self.norm, eps=self.norm_eps,
                            out_dtype=ctx.dtype)
        return ops.gemm(z, self.o_proj)
