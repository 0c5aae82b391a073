"""What a model adds to the residual stream between two layers.

A stretch of layers that runs several times in a row (the same weights, a cache and states of its own for every pass) may
be told which pass it is in: before pass t the vector step[t] is added to every row, and before every pass but the
first the rows as the embedding gave them are added again.  The part is one such place: the vector's row and whether
the embedding's rows come with it; the add happens in the kernel that closes the layer before, ahead of the next norm.
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


register_part("stream_add", "pass_step", PassStep)
