"""What a model adds to the residual stream between two layers.

A stretch of layers that runs several times in a row (the same weights, a cache and states of its own for every pass) may
be told which pass it is in: before pass t the vector step[t] is added to every row, and before every pass but the
first the rows as the embedding gave them are added again.  The part is one such place: the vector's row and whether
the embedding's rows come with it; the add happens in the kernel that closes the layer before, ahead of the next norm.

Or the stream itself may be made anew before every pass: x <- W [x; x0], x0 being the embedding's rows (`StreamMix`).  The
kernel that closes the layer before writes the product's operand rows, and the one that takes the product's sums up as the
new stream applies the next norm.  The stream is float32; a bfloat16 engine multiplies it in two bfloat16 terms (its rounding
and the remainder's rounding, W standing twice side by side), so that what passes keeps 16 bits.
"""
from ..models.spec import TensorSpec
from ..registry import register_part
from .base import StreamAdd


class PassStep(StreamAdd):
    def __init__(self, size, passes, index, origin=False, tensor="step"):
        """tensor: local name of the vectors [passes, size], of which row `index` is added; origin: the embedding's rows too."""
        if not 0 <= index < passes:
            raise ValueError(f"pass {index} of {passes}")
        self.size, self.passes, self.index, self.needs_origin, self.tensor = int(size), int(passes), int(index), bool(origin), tensor

    def tensor_specs(self):
        return {self.tensor: TensorSpec((self.passes, self.size), init="norm")}

    def bind(self, tensors, rt):
        self.rt = rt
        self.vec = tensors[self.tensor][self.index].float().contiguous()

    def operands(self, ctx):
        return self.vec, ctx.origin if self.needs_origin else None


class StreamMix(StreamAdd):
    needs_origin = True
    replaces = True              # the product's rows become the stream

    def __init__(self, size, tensor="in", origin_terms=1):
        """tensor: local name of W [size, 2 size], the stream's columns first.  origin_terms: bfloat16 terms of the embedding's
        rows (one is exact where they are rows of a bfloat16 table as they stand)."""
        self.size, self.tensor, self.origin_terms = int(size), tensor, int(origin_terms)

    def tensor_specs(self):
        return {self.tensor: TensorSpec((self.size, 2 * self.size))}

    def bind(self, tensors, rt):
        import torch
        self.rt = rt
        w = rt.matrix(tensors[self.tensor])
        if w.dtype != torch.float32:
            x, o = w[:, :self.size], w[:, self.size:]
            w = torch.cat([x, x] + [o] * self.origin_terms, dim=1)
        self.w = w.contiguous()

    def forward(self, ctx, stream, a, b, wa, wb, gain, eps, dtype):
        """stream <- W [stream + wa a + wb b; embedding's rows]; returns its norm (or None without a gain)."""
        import torch
        ops = ctx.ops
        rows = ops.join_rms_norm(stream, a, b, None, 0.0, self.w.dtype, origin=ctx.origin, wa=wa, wb=wb, stack=self.origin_terms)
        mixed = ops.linear(rows, self.w, torch.float32, defer=True)
        return ops.join_rms_norm(stream, mixed, None, gain, eps, dtype, fresh=True)


register_part("stream_add", "stream_mix", StreamMix)
register_part("stream_add", "pass_step", PassStep)
