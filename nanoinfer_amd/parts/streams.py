"""Parts around several streams a token: the block whose sublayers read a weighted sum of the streams and whose outputs
are added to all of them while the streams mix, the norm whose weight is stored as its difference from one, and the
feed-forward without a gate.

Kinds registered here: norm ``rmsnorm_one_plus``; stream_link ``static``; feed_forward ``relu2_mlp``; block
``linked_streams``.  Every size and constant is a parameter of the part's spec.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from .. import kernels as K
from ..registry import register_part
from .base import Block, LayerCache, Part, WeightRequest
from .standard import RMSNorm


# ------------------------------------------------------------------ norm

@register_part("norm", "rmsnorm_one_plus")
class OnePlusRMSNorm(RMSNorm):
    """``x * rsqrt(mean(x^2) + eps) * (1 + w)`` in float32.  params: size, eps.  weights: weight [size] = w.  The device
    holds ``1 + w``, so the kernels of norms with a plain weight serve it."""

    def __init__(self, spec, weights, rt):
        super().__init__(spec, {"weight": weights["weight"].to(torch.float32) + 1.0}, rt)


# ------------------------------------------------------------------ what ties a sublayer to the streams

@register_part("stream_link", "static")
class StaticStreamLink(Part):
    """How a sublayer reads from and writes to the streams ``x_1 .. x_s`` of a token: it is given ``sum_s in[s] x_s``, and
    with its output y ``x_t <- sum_f mix[f, t] x_f + out[t] y``, all new streams from the old ones.  params: streams.
    weights: in [streams], out [streams], mix [streams, streams] (indexed [from, to])."""

    graph_safe = True

    @classmethod
    def weight_requests(cls, spec):
        s, w = spec.params["streams"], spec.weights
        return [WeightRequest(w["in"], (s,)), WeightRequest(w["out"], (s,)), WeightRequest(w["mix"], (s, s))]

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        self.streams = int(spec.params["streams"])
        if not 1 <= self.streams <= K.LINK_STREAMS_MAX:
            raise ValueError(f"{self.streams} streams: 1 to {K.LINK_STREAMS_MAX} are compiled")
        self.reads, self.adds, self.mix = (weights[k].to(device=rt.device, dtype=torch.float32).contiguous() for k in ("in", "out", "mix"))


@dataclass
class LinkedSum:
    """What a ``linked_streams`` block hands on as ``pending``: the streams ``h`` have not received the output ``y`` of the
    block's last sublayer yet, nor been mixed by its ``link``.  Whoever comes next does both in the pass that makes its own
    input of the streams."""

    y: torch.Tensor               # float32 [T, d] or [n, T, d]: addends
    link: StaticStreamLink

    def add_to(self, h: torch.Tensor) -> torch.Tensor:
        """The sum of the complete streams, float32 [T, d] (``h`` is left as it is)."""
        v = torch.empty(h.shape[0], h.shape[-1], dtype=torch.float32, device=h.device)
        return K.link_streams(h, self.link.streams, self.y, self.link.mix, self.link.adds, None, None, 0.0, v)

    def normed(self, h: torch.Tensor, norm, rows: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
        """``norm`` of the sum of the complete streams for the given rows alone: the last step of a pass."""
        v = torch.empty(rows.shape[0], h.shape[-1], dtype=dtype, device=h.device)
        return K.link_streams(h, self.link.streams, self.y, self.link.mix, self.link.adds, None, norm.weight, norm.eps, v, rows=rows)


# ------------------------------------------------------------------ feed-forward

@register_part("feed_forward", "relu2_mlp")
class SquaredReluMLP(Part):
    """``W_down relu(W_up x)^2``.  params: hidden_size, intermediate_size.  weights: up [I, d], down [d, I]."""

    graph_safe = True

    @classmethod
    def weight_requests(cls, spec):
        p, w = spec.params, spec.weights
        d, i = p["hidden_size"], p["intermediate_size"]
        return [WeightRequest(w["up"], (i, d)), WeightRequest(w["down"], (d, i))]

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        names = spec.weights
        self.w_up = rt.weight(names["up"], weights["up"])
        self.w_down = rt.weight(names["down"], weights["down"])
        K.stream_lib()

    def hidden(self, x) -> torch.Tensor:
        """What the down product takes (for a part that places that product's result itself)."""
        return K.linear_relu2(x, self.w_up)

    def forward(self, x, ctx):
        return K.linear(self.hidden(x), self.w_down, out_dtype=torch.float32)


# ------------------------------------------------------------------ block

@register_part("block", "linked_streams")
class LinkedStreamsBlock(Block):
    """A pre-norm block over ``streams`` float32 streams a token: ``y = mixer(norm1(sum_s in1[s] x_s))``,
    ``x_t <- sum_f mix1[f, t] x_f + out1[t] y``, then the same with the feed-forward and its own link and norm.  ``ffn``,
    ``ffn_norm`` and ``ffn_link`` may be absent together.

    The stream of the model's pass becomes [T, streams, d] here.  A token's streams all start as the embedding's output,
    so ``h`` stays [T, d] until the first sublayer has an output.  The last sublayer's output is never added in a pass of
    its own: one kernel adds it, mixes the streams and makes the next sublayer's normed input (:class:`LinkedSum` carries
    it from block to block and to the model's last norm).  params: streams."""

    ROLES = {"mixer_link": "stream_link", "mixer_norm": "norm", "mixer": "mixer", "ffn_link": "stream_link", "ffn_norm": "norm",
             "ffn": "feed_forward"}
    OPTIONAL = ("ffn_link", "ffn_norm", "ffn")

    @classmethod
    def _roles(cls, spec):
        missing = [r for r in cls.ROLES if r not in spec.parts and r not in cls.OPTIONAL]
        extra = [r for r in spec.parts if r not in cls.ROLES]
        if any(r in spec.parts for r in cls.OPTIONAL):
            missing += [r for r in cls.OPTIONAL if r not in spec.parts]
        if missing or extra:
            raise ValueError(f"a block of kind {spec.kind!r} has the parts {sorted(cls.ROLES)}; "
                             f"missing: {missing}, not known: {extra}")
        return [(r, f) for r, f in cls.ROLES.items() if r in spec.parts]

    def __init__(self, spec, tensors, rt):
        super().__init__(spec, tensors, rt)
        self.streams = int(spec.params["streams"])
        for role in self.roles:
            part = getattr(self, role)
            if role.endswith("_link") and part.streams != self.streams:
                raise ValueError(f"a link of {part.streams} streams in a block of {self.streams}")
            if role.endswith("_norm") and not (hasattr(part, "weight") and hasattr(part, "eps")):
                raise ValueError("a linked_streams block's norms are RMS norms with a weight and an eps")
        K.stream_lib()

    def _enter(self, h, pending: Optional[LinkedSum], link: StaticStreamLink, norm):
        """``(h, x)``: the streams with what they lacked, and the normed input of the sublayer that ``link`` ties to them."""
        x = torch.empty(h.shape[0], h.shape[-1], dtype=self.rt.dtype, device=h.device)
        if pending is None:
            K.link_streams(h, self.streams, None, None, None, link.reads, norm.weight, norm.eps, x)
            return h, x
        out = h if h.dim() == 3 else torch.empty(h.shape[0], self.streams, h.shape[1], dtype=torch.float32, device=h.device)
        K.link_streams(h, self.streams, pending.y, pending.link.mix, pending.link.adds, link.reads, norm.weight, norm.eps, x, h_out=out)
        return out, x

    @staticmethod
    def _left(y, link: StaticStreamLink) -> LinkedSum:
        return LinkedSum((y if y.dtype == torch.float32 else y.to(torch.float32)).contiguous(), link)

    def forward(self, h, pending, ctx, cache: LayerCache):
        if pending is not None and not isinstance(pending, LinkedSum):
            raise K.KernelError("a linked_streams block reads a stream that is complete, or that another such block has left")
        if pending is None and h.dim() != 2:
            raise K.KernelError("the streams of a first block are one row a token")
        h, x = self._enter(h, pending, self.mixer_link, self.mixer_norm)
        pending = self._left(self.mixer.forward(x, ctx, cache), self.mixer_link)
        if "ffn" in self.roles:
            h, x = self._enter(h, pending, self.ffn_link, self.ffn_norm)
            pending = self._left(self.ffn.forward(x, ctx), self.ffn_link)
        return h, pending
