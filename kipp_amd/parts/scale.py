"""Scale parts: what a sublayer's result is multiplied by before it is added to the residual stream.  Interface:

    params(spec), load(tensors)
    apply(delta) -> Pending         the scaled delta, not carried out yet: the norm that follows does it in its own kernel
"""
from __future__ import annotations

from ..runtime import ColumnScaled
from .base import ParamSpec, register


@register("scale", "layer_scale")
class LayerScale:
    """A learned factor a column (`LayerScaleSpec`), applied in float32 on its way into the residual sum."""

    graph_safe = True   # forward launches kernels only: no host reads, no data-dependent launches

    def __init__(self, spec, runtime):
        self.spec = spec
        self.rt = runtime
        self.weight = None

    @staticmethod
    def params(spec):
        return {spec.name: ParamSpec((spec.width,), "float", ("one_plus_normal", 0.2))}

    @staticmethod
    def placement(spec):
        return {spec.name: "float32"}

    def load(self, tensors):
        self.weight = tensors[self.spec.name]

    def apply(self, delta):
        return ColumnScaled(self.rt, delta, self.weight)
