"""A residual of several parallel streams (hyper-connections).  Instead of one row x a token has `streams` rows x_s, all
equal to the embedding's output at the start.  Around each of a block's two parts:

    u = sum_s in[s] x_s;   y = part(norm(u));   x_t <- sum_s mix[s, t] x_s + out[t] y     (all at once, from the old ones)

and what follows the last block reads the streams' sum.  Between two blocks the stream is float32 [T, streams, D]; behind
the embedding it is one row expanded over the streams, which the first update reads as such.  Every update runs in one
kernel with the read and the norm in front of the next part, in this block or the next."""
from __future__ import annotations

import torch

from ..kernels import ops
from ..registry import BLOCKS
from .base import Block, Norm, ParamSpec


class StreamRead(Norm):
    """norm(sum_s weights[s] x_s) of a [T, S, D] residual, as the norm that a block applies first."""

    def __init__(self, norm: Norm):
        self.norm = norm
        self.weights: torch.Tensor | None = None   # float32 [S]

    def forward(self, x, out_dtype):
        return ops.streams(x, in_weights=self.weights, weight=self.norm.scale, eps=self.norm.eps, out_dtype=out_dtype)[1]


def begin_streams(x: torch.Tensor, streams: int) -> torch.Tensor:
    """The embedding's output [T, D] as `streams` equal streams (no copy)."""
    return x.unsqueeze(1).expand(-1, streams, -1)


class StreamSum:
    """The end of a model with streams: their sum, alone or with the model's last norm."""

    def __init__(self, streams: int):
        self.streams = int(streams)
        self._ones: torch.Tensor | None = None

    def _weights(self, device) -> torch.Tensor:
        if self._ones is None or self._ones.device != device:
            self._ones = torch.ones(self.streams, dtype=torch.float32, device=device)
        return self._ones

    def to_device(self, device) -> None:
        self._weights(torch.device(device))

    def plain(self, h: torch.Tensor) -> torch.Tensor:
        return ops.streams(h, in_weights=self._weights(h.device))[1]

    def normed_rows(self, h: torch.Tensor, rows: torch.Tensor, norm: Norm, dtype: torch.dtype) -> torch.Tensor:
        if getattr(norm, "fusable_rms", False) and not norm.scale_plus_one:
            return ops.streams(h, in_weights=self._weights(h.device), weight=norm.scale, eps=norm.eps, rows=rows,
                               out_dtype=dtype)[1]
        return norm.forward(ops.streams(h, in_weights=self._weights(h.device), rows=rows)[1], dtype)


@BLOCKS.register("hyper_connections")
class HyperConnectionsBlock(Block):
    """Norms: 'pre_mixer' and, if there is a feed-forward, 'pre_ffn' (RMS norms with a weight that is the gain itself).
    Tensors of the block: 'mixer_in', 'mixer_mix', 'mixer_out' and, with a feed-forward, 'ffn_in', 'ffn_mix', 'ffn_out'."""

    def __init__(self, mixer, feed_forward, norms, streams: int):
        super().__init__(mixer, feed_forward, norms)
        self.streams = int(streams)
        if self.streams < 1:
            raise ValueError("hyper_connections: at least one stream")
        self.sublayers = ("mixer", "ffn") if feed_forward is not None else ("mixer",)
        self.reads: dict[str, StreamRead] = {}
        for q in self.sublayers:
            norm = self.norms.get("pre_" + q)
            if norm is None:
                raise ValueError(f"hyper_connections block: norms missing: ['pre_{q}']")
            if not getattr(norm, "fusable_rms", False) or norm.scale_plus_one:
                raise ValueError("hyper_connections: the norms in front of the parts are RMS norms whose weight is the gain")
            self.reads[q] = StreamRead(norm)
        self.mix: dict[str, torch.Tensor] = {}
        self.out: dict[str, torch.Tensor] = {}

    def param_specs(self):
        S, vec = self.streams, dict(role="vector", init="norm")
        specs = {}
        for q in self.sublayers:
            specs.update({q + "_in": ParamSpec((S,), **vec), q + "_mix": ParamSpec((S, S), **vec),
                          q + "_out": ParamSpec((S,), **vec)})
        return specs

    def load(self, tensors):
        for q in self.sublayers:
            self.reads[q].weights = tensors[q + "_in"].to(torch.float32).contiguous()
            self.mix[q] = tensors[q + "_mix"].to(torch.float32).contiguous()
            self.out[q] = tensors[q + "_out"].to(torch.float32).contiguous()

    def first_norm(self):
        return self.reads["mixer"]

    def _write(self, h, y, q, read, dtype):
        """The streams after part `q` returned y, and what `read` reads from them (None: nothing)."""
        if read is not None and not isinstance(read, StreamRead):
            raise TypeError("hyper_connections: a block of one stream cannot follow a block of several")
        weights = (None, None, 0.0) if read is None else (read.weights, read.norm.scale, read.norm.eps)
        return ops.streams(h, y=y, mix=self.mix[q], out_weights=self.out[q], in_weights=weights[0], weight=weights[1],
                           eps=weights[2], out_dtype=dtype)

    def forward(self, h, ctx, cache, normed, next_norm):
        def run(part, x, *args):
            return part.forward(x, ctx, *args, **({"defer_sum": True} if part.defers_sum and ctx.dtype == torch.bfloat16 else {}))

        if normed is None:
            normed = self.reads["mixer"].forward(h, ctx.dtype)
        y = run(self.mixer, normed, cache)
        if self.feed_forward is None:
            return self._write(h, y, "mixer", next_norm, ctx.dtype)
        h, normed = self._write(h, y, "mixer", self.reads["ffn"], ctx.dtype)
        return self._write(h, run(self.feed_forward, normed), "ffn", next_norm, ctx.dtype)
