"""What follows the sublayers of a layer whose result is averaged over the depths, and its dense feed-forward.

Recorded in FLOAT, as `streams` is."""
from .. import ops
from .base_layer import BaseLayer
from .state_space import tensor
from .streams import NamedLinear, WeightNorm


class SquaredReLU(BaseLayer):
    """W_down relu(W_up h)^2."""

    def __init__(self, context, name, width, ff):
        super().__init__(context, name)
        self.up, self.down = NamedLinear(self.context, "up", width, ff), NamedLinear(self.context, "down", ff, width)

    def __call__(self, graph, h, layer_id=None):
        with graph.nameScope(self.context):
            u = ops.relu(graph, self.up(graph, h))
            return self.down(graph, ops.mul(graph, u, u))


class TokenInput(BaseLayer):
    """x + norm(proj(gelu(gate x) * e)), e being the token's own row of this layer: tensors `<context>.gate`, `.proj`, `.norm`."""

    def __init__(self, context, name, width, dim, eps):
        super().__init__(context, name)
        self.gate, self.proj = NamedLinear(self.context, "gate", width, dim), NamedLinear(self.context, "proj", dim, width)
        self.norm = WeightNorm(self.context, "norm", width, eps, centred=False)

    def __call__(self, graph, x, e):
        with graph.nameScope(self.context):
            g = ops.mul(graph, ops.gelu(graph, self.gate(graph, x)), e)
            return ops.add(graph, x, self.norm(graph, self.proj(graph, g)))


class DepthAverage(BaseLayer):
    """The weighted sum of the residuals of all depths: tensor `<context>` [depths]."""

    def __init__(self, context, name, depths):
        super().__init__(context, name)
        self.depths = depths
        self.weight_id = tensor(self, self.context, [depths])

    def __call__(self, graph, history):
        with graph.nameScope(self.context):
            weights = ops.split(graph, self.weight_id, self.depths, axis=0, splits=[1] * self.depths, name="split_weights")
            return ops.sum_op(graph, [ops.mul(graph, x, w) for x, w in zip(history, weights)])
