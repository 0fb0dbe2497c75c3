"""Layers of decoders with attention by heads and feed-forwards that may be mixtures of experts: what a HeadMixer describes, and
the feed-forwards.

Recorded in FLOAT, as `streams` is."""
import numpy as np

from .. import ops
from .base_layer import BaseLayer
from .streams import NamedLinear, WeightNorm, rms_normalised, scalar

HIDDEN = -1e30


def numbers(graph, values, name):
    """Exact numbers that an executor reads off the graph."""
    ops.constant(graph, np.array(values, np.float64), name)


class VisibleKeys(BaseLayer):
    """What is added to the scores of position `step`: a row of a table [positions, rows of the cache, newest first]."""

    def __init__(self, name, positions, rows, mixer):
        super().__init__(None, name)
        table = np.where(mixer.visible(positions)[:, :rows], 0.0, HIDDEN).astype(np.float32)
        self.table_id = self.add_initialized_input_tensor(table, name)
        self.rows = rows

    def __call__(self, graph, step):
        return ops.reshape(graph, ops.dynamic_slice(graph, self.table_id, step, axes=[0], sizes=[1]), [1, 1, 1, self.rows])


class HeadAttention(BaseLayer):
    """Attention over cached keys and values by heads (a HeadMixer): tensors `<context>.q`, `.k`, `.v` with biases where it has
    them, `.q.norm`, `.k.norm`, `.sink`, `.g`, `.o`, and of two maps `.lq1`, `.lk1`, `.lq2`, `.lk2`."""

    def __init__(self, context, name, width, eps, mixer, rotation, visible):
        super().__init__(context, name)
        m = self.mixer = mixer
        self.rotation, self.visible, self.eps = rotation, visible, eps
        self.q, self.k = (NamedLinear(self.context, n, width, h * m.maps * m.dim, n in m.biases) for n, h in (("q", m.heads), ("k", m.kv_heads)))
        self.v = None if m.keys_are_values else NamedLinear(self.context, "v", width, m.kv_heads * m.vdim, "v" in m.biases)
        self.q_norm, self.k_norm = (WeightNorm(self.context, n, m.dim, eps, centred=False) for n in ("q.norm", "k.norm"))
        self.g = None
        if m.gate is not None:
            self.g = NamedLinear(self.context, "g", width, m.heads if m.gate == "head" else m.heads * m.vdim)
        self.sink_id = self._vector("sink", m.heads) if m.sink else None
        if m.diff is not None:
            self.lambda_ids = [self._vector(n, m.dim) for n in ("lq1", "lk1", "lq2", "lk2")]
        self.o = NamedLinear(self.context, "o", m.heads * m.vdim, width)

    def _vector(self, name, size):
        key = f"{self.context}.{name}"
        return self.add_initialized_input_tensor(np.asarray(self.get_param_from_state_dict(key, [size]), np.float32), key)

    def _normed(self, graph, norm, x, step, heads):
        m = self.mixer
        x = norm(graph, ops.reshape(graph, x, [self.batch_size, heads * m.maps, m.dim]))
        return x if self.rotation is None else self.rotation(graph, x, step, m.dim)

    def _weight_of_second(self, graph):
        a1, b1, a2, b2 = self.lambda_ids
        one, two = (ops.exp(graph, ops.reduce_sum(graph, ops.mul(graph, a, b), axes=[0], keepdims=True)) for a, b in ((a1, b1), (a2, b2)))
        return ops.add(graph, ops.sub(graph, one, two), scalar(graph, self.mixer.diff, "diff"))

    def __call__(self, graph, h, layer_id, step):
        m, B, W = self.mixer, self.batch_size, self.visible.rows
        G, R, M, D, E = m.kv_heads, m.heads // m.kv_heads, m.maps, m.dim, m.vdim
        with graph.nameScope(self.context):
            numbers(graph, m.numbers(), f"l{layer_id}.mixer")
            if m.rot is not None:
                numbers(graph, m.rot.numbers(), f"l{layer_id}.rotation")
            k = self.k(graph, h)
            v = ops.reshape(graph, k if self.v is None else self.v(graph, h), [B, G, 1, E])
            q = self._normed(graph, self.q_norm, self.q(graph, h), step, m.heads)
            k = ops.reshape(graph, self._normed(graph, self.k_norm, k, step, G), [B, G * M, 1, D])
            keys = ops.transpose(graph, ops.kv_cache(graph, step, k, W, 2, 1), [0, 1, 3, 2])            # newest first
            values = ops.kv_cache(graph, step, v, W, 2, 1)
            q = ops.transpose(graph, ops.reshape(graph, q, [B, G, R, M, D]), [0, 1, 3, 2, 4])
            s = ops.mul(graph, ops.matmul(graph, ops.reshape(graph, q, [B, G * M, R, D]), keys), scalar(graph, m.scale, "score_scale"))
            s = ops.add(graph, s, self.visible(graph, step))
            if self.sink_id is not None:
                sinks = ops.tile(graph, ops.reshape(graph, self.sink_id, [1, G, R, 1]), [B, 1, 1, 1])
                s = ops.concat(graph, s, sinks, 3)
            p = ops.softmax_ce(graph, s, -1, stable_mode=True)
            if self.sink_id is not None:
                p = ops.static_slice(graph, p, [0], [W], [3])
            o = ops.matmul(graph, ops.reshape(graph, p, [B, G, M * R, W]), values)
            if m.diff is not None:
                a1, a2 = ops.split(graph, ops.reshape(graph, o, [B, G, 2, R * E]), 2, axis=2, splits=[1, 1], name="split_maps")
                o = ops.sub(graph, a1, ops.mul(graph, a2, self._weight_of_second(graph)))
                o = rms_normalised(graph, ops.reshape(graph, o, [B, m.heads, E]), self.eps)
                o = ops.mul(graph, o, scalar(graph, 1.0 - m.diff, "rest_of_diff"))
            if m.gate == "head":
                o = ops.mul(graph, ops.reshape(graph, o, [B, m.heads, E]), ops.reshape(graph, ops.sigmoid(graph, self.g(graph, h)), [B, m.heads, 1]))
            o = ops.reshape(graph, o, [B, 1, m.heads * E])
            if m.gate == "feature":
                o = ops.mul(graph, o, ops.sigmoid(graph, self.g(graph, h)))
            return self.o(graph, o)


class SwiGLU(BaseLayer):
    """W_down (silu(W_gate h) * (W_up h))."""

    def __init__(self, context, name, width, ff):
        super().__init__(context, name)
        self.gate, self.up = (NamedLinear(self.context, n, width, ff) for n in ("gate", "up"))
        self.down = NamedLinear(self.context, "down", ff, width)

    def activated(self, graph, g, u):
        return ops.mul(graph, ops.mul(graph, g, ops.sigmoid(graph, g)), u)

    def __call__(self, graph, h, layer_id=None):
        with graph.nameScope(self.context):
            return self.down(graph, self.activated(graph, self.gate(graph, h), self.up(graph, h)))


class ClampedExpert(SwiGLU):
    """W_down (g sigmoid(slope g) (u + 1)), g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit)."""

    def __init__(self, context, name, width, glu):
        super().__init__(context, name, width, glu.ff)
        self.limit, self.slope = glu.limit, glu.slope

    def activated(self, graph, g, u):
        g = ops.clip(graph, g, clip_min=None, clip_max=self.limit)
        u = ops.clip(graph, u, clip_min=-self.limit, clip_max=self.limit)
        g = ops.mul(graph, g, ops.sigmoid(graph, ops.mul(graph, g, scalar(graph, self.slope, "gate_slope"))))
        return ops.mul(graph, g, ops.add(graph, u, scalar(graph, 1.0, "one")))


class ExpertMixture(BaseLayer):
    """The `top` of the experts with the largest router softmax scores, weighted by score * scale, and a shared one weighted by a
    sigmoid: tensors `<context>.router`, `.e<n>.*`, `.shared.*`, `.shared.sg`.  Recorded with every expert at work and weights of
    zero for those that are not chosen."""

    def __init__(self, context, name, width, experts):
        super().__init__(context, name)
        e = self.experts = experts
        self.router = NamedLinear(self.context, "router", width, e.count)
        self.parts = [ClampedExpert(self.context, f"e{n}", width, e.expert) for n in range(e.count)]
        self.shared = None
        if e.shared is not None:
            self.shared = ClampedExpert(self.context, "shared", width, e.shared)
            self.shared_gate = NamedLinear(self.context, "shared.sg", width, 1)

    def weights(self, graph, h):
        """[B, 1, experts]: an expert is chosen when fewer than `top` others score higher."""
        e, B = self.experts, self.batch_size
        s = ops.softmax_ce(graph, self.router(graph, h), -1, stable_mode=True)
        higher = ops.greater(graph, ops.reshape(graph, s, [B, 1, e.count]), ops.reshape(graph, s, [B, e.count, 1]))
        rank = ops.reduce_sum(graph, ops.cast(graph, higher, "FLOAT"), axes=[2], keepdims=False)
        chosen = ops.cast(graph, ops.less(graph, rank, scalar(graph, e.top, "top")), "FLOAT")
        return ops.mul(graph, ops.mul(graph, s, ops.reshape(graph, chosen, [B, 1, e.count])), scalar(graph, e.scale, "router_scale"))

    def __call__(self, graph, h, layer_id):
        e = self.experts
        with graph.nameScope(self.context):
            numbers(graph, [e.count, e.top, e.scale, e.expert.limit, *(() if e.shared is None else (e.shared.limit,))], f"l{layer_id}.experts")
            w = self.weights(graph, h)
            columns = [w] if e.count == 1 else ops.split(graph, w, e.count, axis=2, splits=[1] * e.count, name="split_weights")
            terms = [ops.mul(graph, part(graph, h), c) for part, c in zip(self.parts, columns)]
            if self.shared is not None:
                terms.append(ops.mul(graph, self.shared(graph, h), ops.sigmoid(graph, self.shared_gate(graph, h))))
            return ops.sum_op(graph, terms)
