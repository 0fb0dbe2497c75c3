"""Layers of decoders with attention by heads and feed-forwards that may be mixtures of experts: what a HeadMixer describes, and
the feed-forwards.

Recorded in FLOAT, as `streams` is."""
import numpy as np

from .. import ops
from ..engine.hybrid import ClampedGLU
from .base_layer import BaseLayer
from .state_space import ShortConvolution, tensor
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
    them and their `.conv`, `.q.norm`, `.k.norm`, `.sink`, `.r1`, `.r2`, `.g`, `.o`, and of two maps `.lq1`, `.lk1`, `.lq2`, `.lk2`."""

    def __init__(self, context, name, width, eps, mixer, rotation, visible):
        super().__init__(context, name)
        m = self.mixer = mixer
        self.rotation, self.visible, self.eps = rotation, visible, eps
        self.q, self.k = (NamedLinear(self.context, n, width, h * m.maps * m.dim, n in m.biases) for n, h in (("q", m.heads), ("k", m.kv_heads)))
        self.v = None if m.keys_are_values else NamedLinear(self.context, "v", width, m.kv_heads * m.vdim, "v" in m.biases)
        self.q_norm = self.k_norm = None
        if m.norms:
            self.q_norm, self.k_norm = (WeightNorm(self.context, n, m.dim, eps, centred=False) for n in ("q.norm", "k.norm"))
        self.convs = [ShortConvolution(self.context, f"{n}.conv", h, m.taps) for n, h in
                      (("q", m.heads * m.maps * m.dim), ("k", m.kv_heads * m.maps * m.dim), ("v", m.kv_heads * m.vdim))] if m.taps else []
        self.far_ids = [self._vector(n, m.heads) for n in ("r1", "r2")] if m.far else None
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

    def state_shapes(self):
        """Of what the loop carries: the convolutions' rows"""
        return [c.state_shape() for c in self.convs]

    def _normed(self, graph, norm, x, step, heads):
        m = self.mixer
        x = ops.reshape(graph, x, [self.batch_size, heads * m.maps, m.dim])
        x = x if norm is None else norm(graph, x)
        return x if self.rotation is None else self.rotation(graph, x, step, m.dim)

    def _weight_of_second(self, graph):
        a1, b1, a2, b2 = self.lambda_ids
        one, two = (ops.exp(graph, ops.reduce_sum(graph, ops.mul(graph, a, b), axes=[0], keepdims=True)) for a, b in ((a1, b1), (a2, b2)))
        return ops.add(graph, ops.sub(graph, one, two), scalar(graph, self.mixer.diff, "diff"))

    def _penalty(self, graph):
        """[1, G, R, W]: what the distances of the cache's rows, newest first, take off the heads' scores"""
        m, W = self.mixer, self.visible.rows
        r1, r2 = (ops.reshape(graph, t, [1, m.kv_heads, m.heads // m.kv_heads, 1]) for t in self.far_ids)
        back = ops.constant(graph, np.arange(W, dtype=np.float32).reshape(1, 1, 1, W), "distances")
        return ops.mul(graph, r1, ops.log(graph, ops.add(graph, ops.mul(graph, r2, back), scalar(graph, 1.0, "one"))))

    def __call__(self, graph, h, layer_id, step, state=()):
        """The result; with short convolutions (result, state for the next token)"""
        m, B, W = self.mixer, self.batch_size, self.visible.rows
        G, R, M, D, E = m.kv_heads, m.heads // m.kv_heads, m.maps, m.dim, m.vdim
        with graph.nameScope(self.context):
            numbers(graph, m.numbers(), f"l{layer_id}.mixer")
            if m.rot is not None:
                numbers(graph, m.rot.numbers(), f"l{layer_id}.rotation")
            q, k = self.q(graph, h), self.k(graph, h)
            v = k if self.v is None else self.v(graph, h)
            if self.convs:
                (q, a), (k, b), (v, c) = (conv(graph, t, before) for conv, t, before in zip(self.convs, (q, k, v), state))
                state = [a, b, c]
            v = ops.reshape(graph, v, [B, G, 1, E])
            q = self._normed(graph, self.q_norm, q, step, m.heads)
            k = ops.reshape(graph, self._normed(graph, self.k_norm, k, step, G), [B, G * M, 1, D])
            keys = ops.transpose(graph, ops.kv_cache(graph, step, k, W, 2, 1), [0, 1, 3, 2])            # newest first
            values = ops.kv_cache(graph, step, v, W, 2, 1)
            q = ops.transpose(graph, ops.reshape(graph, q, [B, G, R, M, D]), [0, 1, 3, 2, 4])
            s = ops.mul(graph, ops.matmul(graph, ops.reshape(graph, q, [B, G * M, R, D]), keys), scalar(graph, m.scale, "score_scale"))
            s = ops.add(graph, s, self.visible(graph, step))
            if self.far_ids is not None:
                s = ops.sub(graph, s, self._penalty(graph))
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
            o = self.o(graph, o)
            return (o, state) if self.convs else o


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
    """The `top` of the experts with the largest router scores and what else an Experts describes, and a shared one weighted by a
    sigmoid: tensors `<context>.router`, `.correction`, `.e<n>.*`, `.shared.*`, `.shared.sg`.  Recorded with every expert at work and
    weights of zero for those that are not chosen."""

    def __init__(self, context, name, width, experts):
        super().__init__(context, name)
        e = self.experts = experts
        self.router = NamedLinear(self.context, "router", width, e.count)
        clamped = isinstance(e.expert, ClampedGLU)
        self.parts = [ClampedExpert(self.context, f"e{n}", width, e.expert) if clamped else SwiGLU(self.context, f"e{n}", width, e.expert.ff)
                      for n in range(e.count)]
        self.limits = [x.limit for x in (e.expert, e.shared) if x is not None] if clamped else None
        self.correction_id = tensor(self, f"{self.context}.correction", [e.count]) if e.corrected else None
        self.shared = None
        if e.shared is not None:
            self.shared = ClampedExpert(self.context, "shared", width, e.shared)
            self.shared_gate = NamedLinear(self.context, "shared.sg", width, 1)

    def weights(self, graph, h):
        """[B, 1, experts]: an expert is chosen when fewer than `top` others score higher."""
        e, B = self.experts, self.batch_size
        z = self.router(graph, h)
        s = ops.sigmoid(graph, z) if e.score == "sigmoid" else ops.softmax_ce(graph, z, -1, stable_mode=True)
        choice = s if self.correction_id is None else ops.add(graph, s, self.correction_id)

        def best(scores, n, count, groups=1):
            """1 for the `count` largest of each group's n scores, else 0; [B, groups, n]"""
            higher = ops.greater(graph, ops.reshape(graph, scores, [B, groups, 1, n]), ops.reshape(graph, scores, [B, groups, n, 1]))
            rank = ops.reduce_sum(graph, ops.cast(graph, higher, "FLOAT"), axes=[3], keepdims=False)
            return ops.cast(graph, ops.less(graph, rank, scalar(graph, count, "count")), "FLOAT")
        if e.keep < e.groups:
            size = e.count // e.groups
            two = ops.mul(graph, ops.reshape(graph, choice, [B, e.groups, size]), best(choice, size, 2, e.groups))
            kept = best(ops.reduce_sum(graph, two, axes=[2], keepdims=False), e.groups, e.keep)
            closed = ops.mul(graph, ops.sub(graph, kept, scalar(graph, 1.0, "one")), scalar(graph, -HIDDEN, "hidden"))
            choice = ops.add(graph, ops.reshape(graph, choice, [B, e.groups, size]), ops.reshape(graph, closed, [B, e.groups, 1]))
        w = ops.mul(graph, s, ops.reshape(graph, best(choice, e.count, e.top), [B, 1, e.count]))
        if e.share:
            total = ops.add(graph, ops.reduce_sum(graph, w, axes=[2], keepdims=True), scalar(graph, 1e-20, "share_eps"))
            w = ops.div(graph, w, total)
        return ops.mul(graph, w, scalar(graph, e.scale, "router_scale"))

    def __call__(self, graph, h, layer_id):
        e = self.experts
        with graph.nameScope(self.context):
            numbers(graph, e.numbers(), f"l{layer_id}.experts")
            if self.limits is not None:
                numbers(graph, self.limits, f"l{layer_id}.limits")
            w = self.weights(graph, h)
            columns = [w] if e.count == 1 else ops.split(graph, w, e.count, axis=2, splits=[1] * e.count, name="split_weights")
            terms = [ops.mul(graph, part(graph, h), c) for part, c in zip(self.parts, columns)]
            if self.shared is not None:
                terms.append(ops.mul(graph, self.shared(graph, h), ops.sigmoid(graph, self.shared_gate(graph, h))))
            return ops.sum_op(graph, terms)
