"""Layers of decoders whose sublayers stand side by side on one residual: norm in groups, token shift, gated results.

Recorded in FLOAT, as `streams` is."""
import numpy as np

from .. import ops
from .base_layer import BaseLayer
from .streams import NamedLinear, WeightNorm, rms_normalised


class GroupedRMSNorm(WeightNorm):
    """RMS norm of each of `groups` equal consecutive parts, one weight over the whole: tensor `<context>` [size]."""

    def __init__(self, context, name, size, eps, groups):
        if size % groups:
            raise ValueError(f"{groups} groups do not divide a width of {size}")
        super().__init__(context, name, size, eps, centred=False)
        self.groups = groups

    def __call__(self, graph, x):
        B = self.batch_size
        with graph.nameScope(self.context):
            parts = ops.reshape(graph, x, [B, 1, self.groups, self.size // self.groups])
            whole = ops.reshape(graph, rms_normalised(graph, parts, self.eps), [B, 1, self.size])
            return ops.mul(graph, whole, self.weight_id)


class TokenShift(BaseLayer):
    """h + (h_before - h) * mix with tensor `<context>` [size]; h_before is carried by the loop and starts as zeros."""

    def __init__(self, context, name, size):
        super().__init__(context, name)
        self.size = size
        self.collect_bind_layer_weights()

    def collect_bind_layer_weights(self):
        mix = np.asarray(self.get_param_from_state_dict(self.context, [self.size]), np.float32)
        self.mix_id = self.add_initialized_input_tensor(mix, self.context)

    def state_shape(self):
        return [self.batch_size, 1, self.size]

    def __call__(self, graph, h, before):
        """(what the sublayer reads, what the next token finds)"""
        with graph.nameScope(self.context):
            return ops.add(graph, h, ops.mul(graph, ops.sub(graph, before, h), self.mix_id)), h


class ResultGate(BaseLayer):
    """A sublayer's result times sigmoid(W h + b): tensors `<context>` [size, size] and `<context>.b` [size]."""

    def __init__(self, context, name, size):
        super().__init__(context, name)
        self.linear = NamedLinear(context, name, size, size, use_bias=True)

    def __call__(self, graph, h, y):
        return ops.mul(graph, y, ops.sigmoid(graph, self.linear(graph, h)))


class BiasedSwiGLU(BaseLayer):
    """W_down (silu(W_gate h + b) * (W_up h + b)) + b."""

    def __init__(self, context, name, width, ff, kind="dense"):
        super().__init__(context, name)
        if kind != "dense":
            raise ValueError(f"Invalid feed-forward {kind}, options: ['dense']")
        self.gate, self.up = (NamedLinear(self.context, n, width, ff, use_bias=True) for n in ("gate", "up"))
        self.down = NamedLinear(self.context, "down", ff, width, use_bias=True)

    def __call__(self, graph, h):
        with graph.nameScope(self.context):
            g = self.gate(graph, h)
            g = ops.mul(graph, g, ops.sigmoid(graph, g))
            return self.down(graph, ops.mul(graph, g, self.up(graph, h)))


class RotaryTable(BaseLayer):
    """cos and sin of every position, [positions, dims / 2] each, for features i and i + dims / 2 turned together, or
    (`neighbours`) features 2 i and 2 i + 1.  Frequencies other than base^(-2 i / dims), and a factor of both, may be given."""

    def __init__(self, name, positions, base, dims, neighbours=False, frequencies=None, amplitude=1.0):
        super().__init__(None, name)
        self.dims, self.neighbours = dims, neighbours
        f = float(base) ** (-2.0 * np.arange(dims // 2) / dims) if frequencies is None else frequencies
        angle = np.arange(positions)[:, None] * f
        self.ids = [self.add_initialized_input_tensor((f(angle) * amplitude).astype(np.float32), f"{name}.{n}")
                    for f, n in ((np.cos, "cos"), (np.sin, "sin"))]

    def __call__(self, graph, x, step, size):
        """x [B, n, size], its first `dims` features turned by the angles of position `step`."""
        half, rest = self.dims // 2, size - self.dims
        cos, sin = (ops.reshape(graph, ops.dynamic_slice(graph, t, step, axes=[0], sizes=[1]), [1, 1, half]) for t in self.ids)
        if self.neighbours:
            return self._neighbours(graph, x, cos, sin, size)
        parts = [half, half] + ([rest] if rest else [])
        u, v, *tail = ops.split(graph, x, len(parts), axis=2, splits=parts, name="split_rotated")
        a = ops.sub(graph, ops.mul(graph, u, cos), ops.mul(graph, v, sin))
        b = ops.add(graph, ops.mul(graph, v, cos), ops.mul(graph, u, sin))
        y = ops.concat(graph, a, b, 2)
        return ops.concat(graph, y, tail[0], 2) if tail else y

    def _neighbours(self, graph, x, cos, sin, size):
        half, rest = self.dims // 2, size - self.dims
        B, n = self.batch_size, -1
        turned = x
        if rest:
            turned, tail = ops.split(graph, x, 2, axis=2, splits=[self.dims, rest], name="split_rotated")
        u, v = ops.split(graph, ops.reshape(graph, turned, [B, n, half, 2]), 2, axis=3, splits=[1, 1], name="split_neighbours")
        u, v = (ops.squeeze(graph, t, [3]) for t in (u, v))
        a = ops.sub(graph, ops.mul(graph, u, cos), ops.mul(graph, v, sin))
        b = ops.add(graph, ops.mul(graph, v, cos), ops.mul(graph, u, sin))
        y = ops.reshape(graph, ops.concat(graph, ops.unsqueeze(graph, a, [3]), ops.unsqueeze(graph, b, [3]), 3), [B, n, self.dims])
        return ops.concat(graph, y, tail, 2) if rest else y
