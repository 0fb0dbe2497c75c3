"""The state-space recurrence of Mamba-2, and the short convolution ahead of it (and of other mixers).

Recorded in FLOAT, as `streams` is."""
import numpy as np

from .. import ops
from .base_layer import BaseLayer
from .streams import NamedLinear, rms_normalised


def tensor(layer, name, shape):
    """The tensor of that name, which belongs to `layer`."""
    return layer.add_initialized_input_tensor(np.asarray(layer.get_param_from_state_dict(name, shape), np.float32), name)


class ShortConvolution(BaseLayer):
    """Causal convolution over `taps` tokens, channel by channel: tensor `<context>` [channels, taps], the last column the current
    token's, and `<context>.b` where there is a bias.  The rows before are carried by the loop, oldest first, and start as zeros."""

    def __init__(self, context, name, channels, taps, bias=False):
        super().__init__(context, name)
        self.channels, self.taps = channels, taps
        self.weight_id = tensor(self, self.context, [channels, taps])
        self.bias_id = tensor(self, f"{self.context}.b", [channels]) if bias else None

    def state_shape(self):
        """None where nothing is carried"""
        return [self.batch_size, self.taps - 1, self.channels] if self.taps > 1 else None

    def __call__(self, graph, x, before):
        """x [B, 1, channels] -> (the convolved row, what the next token finds)"""
        rows = x if before is None else ops.concat(graph, before, x, 1)
        with graph.nameScope(self.context):
            y = ops.mul(graph, rows, ops.transpose(graph, self.weight_id, [1, 0]))
            y = ops.reduce_sum(graph, y, axes=[1], keepdims=True)
            if self.bias_id is not None:
                y = ops.add(graph, y, self.bias_id)
            return y, before if before is None else ops.static_slice(graph, rows, [1], [self.taps], [1])


class StateSpace(BaseLayer):
    """Mamba-2 (a StateSpaceMixer): tensors `<context>.in` (rows z | x | b | c | dt), `.conv`, `.conv.b`, `.dt_bias`, `.A_log`, `.D`,
    `.norm`, `.o`.  State and the convolution's rows are carried by the loop."""

    def __init__(self, context, name, width, eps, mixer):
        super().__init__(context, name)
        m, self.eps = mixer, eps
        self.mixer, self.inner, self.states = m, m.heads * m.vdim, m.groups * m.dim
        self.project = NamedLinear(self.context, "in", width, 2 * self.inner + 2 * self.states + m.heads)
        self.conv = ShortConvolution(self.context, "conv", self.inner + 2 * self.states, m.taps, bias=True)
        self.dt_bias_id, self.a_log_id, self.skip_id = (tensor(self, f"{self.context}.{n}", [m.heads]) for n in ("dt_bias", "A_log", "D"))
        self.norm_id = tensor(self, f"{self.context}.norm", [self.inner])
        self.o = NamedLinear(self.context, "o", self.inner, width)

    def state_shapes(self):
        m = self.mixer
        return [[self.batch_size, m.heads, m.dim, m.vdim], self.conv.state_shape()]

    def __call__(self, graph, h, layer_id, state):
        from .heads import numbers
        m, B, (S, before) = self.mixer, self.batch_size, state
        H, G, N, E = m.heads, m.groups, m.dim, m.vdim
        with graph.nameScope(self.context):
            numbers(graph, m.numbers(), f"l{layer_id}.mixer")
            sizes = [self.inner, self.inner + 2 * self.states, H]
            z, u, dt = ops.split(graph, self.project(graph, h), 3, axis=2, splits=sizes, name="split_projection")
            u, before = self.conv(graph, u, before)
            u = ops.mul(graph, u, ops.sigmoid(graph, u))
            x, b, c = ops.split(graph, u, 3, axis=2, splits=[self.inner, self.states, self.states], name="split_convolved")
            dt = ops.reshape(graph, ops.softplus(graph, ops.add(graph, dt, self.dt_bias_id)), [B, H, 1, 1])
            rate = ops.reshape(graph, ops.exp(graph, self.a_log_id), [1, H, 1, 1])
            keep = ops.reciprocal(graph, ops.exp(graph, ops.mul(graph, rate, dt)))

            def shared(t, shape):
                """a group's row for each of its heads"""
                t = ops.tile(graph, ops.reshape(graph, t, [B, G, 1, N]), [1, 1, H // G, 1])
                return ops.reshape(graph, t, shape)
            x = ops.reshape(graph, x, [B, H, 1, E])
            taken = ops.mul(graph, ops.mul(graph, shared(b, [B, H, N, 1]), dt), x)
            S = ops.add(graph, ops.mul(graph, S, keep), taken)
            y = ops.add(graph, ops.matmul(graph, shared(c, [B, H, 1, N]), S), ops.mul(graph, x, ops.reshape(graph, self.skip_id, [1, H, 1, 1])))
            y = ops.mul(graph, ops.reshape(graph, y, [B, 1, self.inner]), ops.mul(graph, z, ops.sigmoid(graph, z)))
            parts = ops.reshape(graph, y, [B, 1, m.norm_parts, self.inner // m.norm_parts])
            y = ops.reshape(graph, rms_normalised(graph, parts, self.eps), [B, 1, self.inner])
            return self.o(graph, ops.mul(graph, y, self.norm_id)), [S, before]
