"""Layers of decoders with a 32-bit residual in parallel streams: Linears and norms whose tensors are stored under the
layer's own name, and the connection of a sublayer to the streams.

Everything is recorded in FLOAT; which precision the executor multiplies in is the session's precision ('bf16', 'fp32')."""
import numpy as np

from .. import ops
from .base_layer import BaseLayer, require_single_device


def scalar(graph, value, name):
    return ops.constant(graph, np.array(value).astype(np.float32), name)


class NamedLinear(BaseLayer):
    """y = x W^T (+ b): tensor `<context>` [out, in], bias `<context>.b`."""

    def __init__(self, context, name, input_size, output_size, use_bias=False):
        require_single_device("NamedLinear")
        super().__init__(context, name)
        self.input_size, self.output_size, self.use_bias = input_size, output_size, use_bias
        self.collect_bind_layer_weights()

    def collect_bind_layer_weights(self):
        self.weight_id = self.tensor("", [self.output_size, self.input_size])
        if self.use_bias:
            self.bias_id = self.tensor(".b", [self.output_size])

    def tensor(self, suffix, shape):
        key = self.context + suffix
        return self.add_initialized_input_tensor(np.asarray(self.get_param_from_state_dict(key, shape), np.float32), key)

    def __call__(self, graph, x):
        with graph.nameScope(self.context):
            y = ops.matmul(graph, x, ops.transpose(graph, self.weight_id, [1, 0]))
            return ops.add(graph, y, self.bias_id) if self.use_bias else y


def rms_normalised(graph, x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    v = ops.reducemean(graph, ops.mul(graph, x, x))
    return ops.mul(graph, x, ops.reciprocal(graph, ops.sqrt(graph, ops.add(graph, v, scalar(graph, eps, "norm_eps")))))


class WeightNorm(BaseLayer):
    """A norm with a weight and no bias: tensor `<context>` [size].  centred: layer norm, else RMS norm."""

    def __init__(self, context, name, size, eps, centred):
        require_single_device("WeightNorm")
        super().__init__(context, name)
        self.size, self.eps, self.centred = size, eps, centred
        self.collect_bind_layer_weights()

    def collect_bind_layer_weights(self):
        w = np.asarray(self.get_param_from_state_dict(self.context, [self.size]), np.float32)
        self.weight_id = self.add_initialized_input_tensor(w, self.context)

    def __call__(self, graph, x):
        with graph.nameScope(self.context):
            if self.centred:
                x = ops.sub(graph, x, ops.reducemean(graph, x))
            return ops.mul(graph, rms_normalised(graph, x, self.eps), self.weight_id)


class StreamConnection(BaseLayer):
    """Connects one sublayer to S residual streams [S, B * T * d]: it reads sum_s in[s] x_s, and its result y is written
    back as x_t <- sum_s mix[s, t] x_s + mult * out[t] * y, all streams at once.  Tensors `<context>.in`, `.out`, `.mix`
    (from -> to); without them (one plain residual) all are 1."""

    def __init__(self, context, name, streams, mult, plain=False):
        super().__init__(context, name)
        self.streams, self.mult, self.plain = streams, mult, plain
        self.collect_bind_layer_weights()

    def collect_bind_layer_weights(self):
        if self.plain:
            return
        S = self.streams
        self.ids = {}
        for part, shape in (("in", [S]), ("out", [S]), ("mix", [S, S])):
            key = f"{self.context}.{part}"
            self.ids[part] = self.add_initialized_input_tensor(np.asarray(self.get_param_from_state_dict(key, shape), np.float32), key)

    def __call__(self, graph, streams, shape, sublayer):
        with graph.nameScope(self.context):
            if self.plain:
                read = streams
            else:
                read = ops.matmul(graph, ops.reshape(graph, self.ids["in"], [1, self.streams]), streams)
            y = ops.reshape(graph, sublayer(graph, ops.reshape(graph, read, shape)), [1, -1])
            y = ops.mul(graph, y, scalar(graph, self.mult, "residual_mult"))
            if self.plain:
                return ops.add(graph, streams, y)
            kept = ops.matmul(graph, ops.transpose(graph, self.ids["mix"], [1, 0]), streams)
            return ops.add(graph, kept, ops.mul(graph, ops.reshape(graph, self.ids["out"], [self.streams, 1]), y))
