"""Attention through latents: what is kept per token is one row for all heads.

The mixer's input goes down to a query latent c_q = norm(W_dq h) and to [c | r] = W_dkv h, where c (normed) is the
key/value latent and r (rotated) one key part that all heads share.  Head h has the query [q_h | s_h] = W_uq c_q (s_h
rotated), the key [W_uk,h c | r] and the value W_uv,h c.  Since q_h . (W_uk,h c) = (W_uk,h^T q_h) . c and
sum_j p_j W_uv,h c_j = W_uv,h sum_j p_j c_j, the products with W_uk and W_uv move to the queries and to the result:
attention runs with one key head whose rows are [c | r], the values are the rows' first entries, and only those
rows are cached: once as key rows and, because the matrix cores want the keys of a value entry side by side, the
latent once more transposed, as value pages.

Without a query latent (`q_rank` None) the queries are a projection of the mixer's input.
"""
from __future__ import annotations

import torch

from ..config.spec import PartSpec
from ..kernels import ops
from ..registry import MIXERS, POSITION_ENCODINGS
from .base import Mixer, PagedKVNeed, ParamSpec, as_product_weight
from .rope import PartialRoPE


@MIXERS.register("latent_attention")
class LatentAttention(Mixer):
    """Sizes: per head `key_dim` unrotated and `rot_dim` rotated query/key entries and `value_dim` values; latents of
    `q_rank` and `kv_rank` entries, each normed with a weight.  `scale` is the scores' factor as it is.
    `output_gate`, read from the mixer's input: 'head', head h's result is multiplied by sigmoid(W_g h)_h, one number per
    head; 'element', every entry of every head by a number of its own; None.  `position_encoding` over the rot_dim part:
    'pair_rope', or 'partial_rope', whose half-split pairs the projections' rows are reordered for when they are loaded
    (scores do not change when queries and keys are permuted alike), so that the pairs lie side by side in both cases."""

    defers_sum = True

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, rot_dim: int, value_dim: int, q_rank: int | None,
                 kv_rank: int, scale: float, norm_eps: float, window: int | None = None, output_gate: str | None = None,
                 position_encoding: PartSpec | None = None):
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.key_dim, self.rot_dim, self.value_dim = int(key_dim), int(rot_dim), int(value_dim)
        self.q_rank, self.kv_rank = int(q_rank or 0), int(kv_rank)
        self.scale, self.norm_eps, self.output_gate = float(scale), float(norm_eps), output_gate
        if output_gate not in (None, "head", "element"):
            raise ValueError(f"latent_attention: output_gate is None, 'head' or 'element', not {output_gate!r}")
        self.window = int(window) if window else None
        self.position_encoding = (POSITION_ENCODINGS.build(position_encoding.kind, **position_encoding.params)
                                  if position_encoding is not None else None)
        pe = self.position_encoding
        if pe is not None and not hasattr(pe, "frequencies"):
            raise ValueError("latent_attention: the position encoding must give frequencies() (pair_rope, partial_rope)")
        if pe is not None and pe.dims > self.rot_dim:
            raise ValueError(f"latent_attention: {pe.dims} rotated entries in a part of {self.rot_dim}")
        self.in_proj = self.uq_proj = self.o_proj = self.uk_t = self.uv = self.dq_norm = self.dkv_norm = None

    @property
    def gate_width(self) -> int:
        return {None: 0, "head": self.num_heads, "element": self.num_heads * self.value_dim}[self.output_gate]

    def param_specs(self):
        D, H, dk, dr, dv, Rq, R = (self.hidden_size, self.num_heads, self.key_dim, self.rot_dim, self.value_dim,
                                   self.q_rank, self.kv_rank)
        if Rq:
            specs = {"dq_proj": ParamSpec((Rq, D)), "dq_norm": ParamSpec((Rq,), role="vector", init="norm"),
                     "uq_proj": ParamSpec((H * (dk + dr), Rq))}
        else:
            specs = {"q_proj": ParamSpec((H * (dk + dr), D))}
        specs.update({"dkv_proj": ParamSpec((R + dr, D)),
                      "dkv_norm": ParamSpec((R,), role="vector", init="norm"), "uk_proj": ParamSpec((H * dk, R)),
                      "uv_proj": ParamSpec((H * dv, R)), "o_proj": ParamSpec((D, H * dv))})
        if self.output_gate is not None:
            specs["gate_proj"] = ParamSpec((self.gate_width, D))
        return specs

    def _pairs_side_by_side(self, rows: torch.Tensor, unit: int, at: int) -> torch.Tensor:
        """Rows of a projection, `unit` per head with the rotated part from `at` on: half-split pairs (i, i + dims / 2)
        of the rotated part become neighbours (2i, 2i + 1); the rest stays."""
        half = self.position_encoding.dims // 2
        order = torch.arange(unit)
        i = torch.arange(half)
        order[at + 2 * i], order[at + 2 * i + 1] = at + i, at + half + i
        return rows.reshape(-1, unit, rows.shape[1])[:, order.to(rows.device)].reshape(rows.shape)

    def load(self, tensors):
        t = tensors
        H, dk, dv, R = self.num_heads, self.key_dim, self.value_dim, self.kv_rank
        q_name, dkv = ("uq_proj" if self.q_rank else "q_proj"), t["dkv_proj"]
        q_rows = t[q_name]
        if isinstance(self.position_encoding, PartialRoPE):
            q_rows = self._pairs_side_by_side(q_rows, dk + self.rot_dim, dk)
            dkv = self._pairs_side_by_side(dkv, R + self.rot_dim, R)
        rows = [t["dq_proj"] if self.q_rank else q_rows, dkv] + ([t["gate_proj"]] if self.output_gate is not None else [])
        self.in_proj = as_product_weight(torch.cat(rows, dim=0).contiguous())   # rows [c_q or q | c | r | gates]
        self.uq_proj = as_product_weight(q_rows) if self.q_rank else None
        self.o_proj = as_product_weight(t["o_proj"])
        # per head: [kv_rank, key_dim] (W_uk,h transposed: queries go up to the latent) and [value_dim, kv_rank]
        self.uk_t = t["uk_proj"].reshape(H, dk, R).transpose(1, 2).contiguous()
        self.uv = t["uv_proj"].reshape(H, dv, R).contiguous()
        self.dq_norm = t["dq_norm"].contiguous() if self.q_rank else None
        self.dkv_norm = t["dkv_norm"].contiguous()
        if self.position_encoding is not None:
            self.position_encoding.to_device(t["o_proj"].device)

    def cache_need(self):
        return PagedKVNeed(1, self.kv_rank + self.rot_dim, self.window, self.kv_rank)

    def forward(self, x, ctx, cache, defer_sum=False):
        H, dk, dr, dv, Rq, R = self.num_heads, self.key_dim, self.rot_dim, self.value_dim, self.q_rank, self.kv_rank
        group = ctx.groups[cache.group_id]
        pe = self.position_encoding
        freq, rot_dims = pe.frequencies() if pe is not None else (None, 0)
        mult = getattr(pe, "mult", 1.0)
        proj = ops.gemm(x, self.in_proj)
        if self.q_rank:
            cq = ops.rmsnorm(proj[:, :Rq], self.dq_norm, self.norm_eps, False, ctx.dtype)
            q, c_at = ops.gemm(cq, self.uq_proj), Rq                         # [T, H * (dk + dr)]
        else:
            c_at = H * (dk + dr)
            q = proj[:, :c_at]
        qa = ops.head_product(q, self.uk_t, in_stride=dk + dr, tail=dr)      # [T, H * (R + dr)]: [W_uk^T q | s]
        ops.norm_rope_cache_write(qa, ctx.positions, freq, rot_dims, H, 0, R + dr, 0, rot_mult=mult, q_rot_at=R)
        if cache.write:
            # the token's row [norm(c) | rotated r] into the pages
            ops.norm_rope_cache_write(proj[:, c_at:c_at + R + dr], ctx.positions, freq, rot_dims, 0, 1, R + dr, 0,
                                      rot_mult=mult, eps=self.norm_eps, k_weight=self.dkv_norm, k_norm_dims=R,
                                      k_rot_at=R, slot_mapping=group.slot_mapping, k_pages=cache.k_pages,
                                      v_pages=cache.v_pages, key_values=R)
        if ops.attention_maps_units_takes(qa, cache.k_pages, cache.v_pages, H):
            # bfloat16 at sizes that the matrix cores take: units of 16 rows (heads times tokens), keys cut into ranges
            units, few, many, max_q = ctx.attention_units(16 // ops.attention_maps_heads_per_unit(H, 1))
            o = ops.paged_attention_maps_units(qa, cache.k_pages, cache.v_pages, group.block_table, units, 0, few + many,
                                               H, scale=self.scale, window=self.window, max_kv_len=ctx.max_kv_len,
                                               max_q_len=max_q)
        else:
            o = ops.paged_attention_maps(qa, cache.k_pages, cache.v_pages, group.block_table, ctx.token_seq,
                                         ctx.positions, H, scale=self.scale, window=self.window)     # [T, H * R]
        g_at = c_at + R + dr
        o = ops.head_product(o, self.uv,
                             gate=proj[:, g_at:g_at + self.gate_width] if self.output_gate is not None else None)   # [T, H * dv]
        return ops.gemm(o, self.o_proj, defer_sum=defer_sum)
