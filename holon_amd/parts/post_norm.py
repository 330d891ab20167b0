"""A block with a norm on each sublayer's result and none in front of it, over a residual stream kept in float32:

    x += norm1(mixer(x));   x += norm2(ffn(x))

The sublayers read the stream itself (rounded to the engine's dtype). A sublayer's result travels as a `Scaled` term until
the stream is read next: one kernel (`stream_rms_post`, `csrc/parallel_block.hip`) divides it by its root mean square,
multiplies it by the norm's weight, adds it to the rows and leaves them rounded for the next sublayer, or normed by the
model's last norm. A mixer that answers with two terms and their scales (`Pending`) has them summed in that kernel."""
from __future__ import annotations

import torch

from ..registry import register_part
from ..spec import PartRef
from .base import Build, Part, Stream
from .dyt import Scaled
from .parallel_block import mixed_terms


@register_part("block", "postnorm32")
class PostNorm32(Part):
    """x += norm1(mixer(x)); x += norm2(ffn(x)); see the module's text. A layer may lack the feed-forward; its second norm
    is then not built. The norms are of a kind whose weight stands alone behind the division (`output_gain`: `rms32`)."""

    graph_safe = True

    def __init__(self, build: Build, *, layer: int, hidden: int, mixer: PartRef, ffn: PartRef | None,
                 norm: PartRef) -> None:
        super().__init__(build)
        self.hidden = hidden
        self.attach("mixer", build.make(mixer, layer=layer, hidden=hidden))
        self.attach("norm1", build.make(norm, dim=hidden))
        if not hasattr(self.norm1, "output_gain"):
            raise ValueError(f"postnorm32: norm {norm.kind!r} does not say its weight as one vector")
        self.ffn = None
        if ffn is not None:
            self.attach("ffn", build.make(ffn, layer=layer, hidden=hidden))
            self.attach("norm2", build.make(norm, dim=hidden))
        self.gain1 = self.gain2 = None

    def finalize(self) -> None:
        if self.norm1.weight is not None:
            self.gain1 = self.norm1.output_gain(1.0)
            if self.ffn is not None:
                self.gain2 = self.norm2.output_gain(1.0)

    def extra_tensors(self):
        return [g for g in (self.gain1, self.gain2) if g is not None]

    def _rows(self, delta, h: torch.Tensor) -> torch.Tensor:
        """The stream's rows in the engine's dtype, after what waits to be added is added to them."""
        k = self.kernels
        if delta is None:
            return k.narrow_rows(h, self.build.dtype)
        if not isinstance(delta, Scaled):
            raise TypeError("postnorm32: what waits for the stream comes from a block of another kind")
        term, mix = mixed_terms(delta.term)
        gain = delta.gain if delta.gain is not None else delta.norm.output_gain(delta.scale)
        return k.stream_rms_post(h, term, gain, delta.norm.eps, None, 0.0, self.build.dtype, mix)

    def forward(self, stream: Stream, step, site) -> Stream:
        h = stream.h
        if h.dtype != torch.float32 or h is stream.origin:       # the stream becomes float32 rows of its own
            h = stream.h = self.kernels.widen_rows(h)
        a = self._rows(stream.delta, h)
        stream.stats = None
        stream.delta = Scaled(self.mixer(a, step, site), self.norm1, 1.0, self.gain1)
        if self.ffn is not None:
            x = self._rows(stream.delta, h)
            stream.delta = Scaled(self.ffn(x, step), self.norm2, 1.0, self.gain2)
        return stream

    __call__ = forward
