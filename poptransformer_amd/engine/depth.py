"""Executor of decoders whose layers run mixer and feed-forward side by side behind one norm, add the normed projection of the
token's own part of the layer, and go on from an average over all depths:

    x <- x + mixer(n(x)) + ff(n(x));   x <- x + norm(proj(gelu(gate x) * e));   X_{i+1} = x;   x <- sum_j w_j X_j

Layers mix attention over latents, attention by heads and the state-space recurrence; feed-forwards are squared ReLU or mixtures of
experts.  Rows, sequences, sampling and the decode loop are HybridDecoder's.

Launches of a layer in a decode iteration: the mixer's projections, with the dense feed-forward's or a large router's; the mixer's
own (attention with its cache entries, or the recurrence; a short convolution is part of them, passes of many rows run it in a launch
of its own); output projection and the feed-forward's, whose epilogues add to the residual (of a mixture: pairs and downs of the chosen
experts); the experts' weighted sum, rounding; the token's gate; its projection; the end of the layer, which adds, averages, norms and
routes.  The residuals of all depths stay in the row buffers: the mean of a pass reads them once per layer.
"""
from dataclasses import dataclass
from typing import List, Optional

import torch

from .. import _hybrid_lib as H
from .. import hybrid_kernels as HK
from .hybrid import F32, Experts, HybridDecoder
from .mixers import ExpertBuffers, ExpertMixing, HeadMixing, LatentBuffers, LatentMixing, StateSpaceMixing


@dataclass
class DepthLayerWeights:
    norm: torch.Tensor
    proj: HK.WideWeight              # latent: query latent | cache entry | gate; heads: q | k | v; state space: z | x | b | c, tail: dt
    out: HK.WideWeight
    average: torch.Tensor            # fp32 [depths so far]
    side_gate: HK.WideWeight
    side_proj: HK.WideWeight
    side_norm: torch.Tensor
    # latents
    q_norm: Optional[torch.Tensor] = None
    kv_norm: Optional[torch.Tensor] = None
    uq: Optional[HK.WideWeight] = None
    uk_t: Optional[torch.Tensor] = None              # [heads, R, D]
    uv: Optional[torch.Tensor] = None                # [heads, E, R]
    kv: Optional[HK.WideWeight] = None               # keys of all heads | values of all heads, from the latent (None: the sizes are taken absorbed)
    # heads (q_norm, k_norm, sink, lam as in ResultNormLayerWeights)
    proj_bias: Optional[torch.Tensor] = None
    k_norm: Optional[torch.Tensor] = None
    sink: Optional[torch.Tensor] = None
    lam: float = 0.0
    far: Optional[tuple] = None
    conv: Optional[HK.ShortConv] = None              # heads and state space
    # state space
    ssd: Optional[tuple] = None                      # (dt_bias, a_log, skip)
    head_norm: Optional[torch.Tensor] = None
    # feed-forward
    up: Optional[HK.WideWeight] = None
    down: Optional[HK.WideWeight] = None
    ff: object = None                                # a mixture's routed experts (FeedForwardWeights)
    shared: object = None
    router: Optional[torch.Tensor] = None
    router_linear: Optional[HK.WideWeight] = None
    correction: Optional[torch.Tensor] = None
    top: int = 0

    def linears(self):
        """Every weight that all rows go through, once."""
        return [w for w in (self.proj, self.uq, self.out, self.up, self.down, self.side_gate, self.side_proj) if w is not None]

    def active_parameters(self):
        """Parameters of the products that one row goes through."""
        n = sum((w.n_main + w.tail) * w.K for w in self.linears())
        n += sum(t.numel() for t in (self.uk_t, self.uv) if t is not None)
        return n + sum(self.top * w.n_main * w.K for w in (self.ff.linears() if self.ff else ()))


@dataclass
class DepthWeights:
    embed: torch.Tensor
    side: torch.Tensor               # [vocab, layers, features up to a multiple of eight]
    layers: List[DepthLayerWeights]
    final_norm: torch.Tensor
    head: HK.WideWeight

    def nbytes(self, rows=1):
        """Bytes of the weights that a pass of `rows` rows reads: of a mixture the experts that so many choose on average, where every
        choice is as likely as another."""
        n = self.head.nbytes
        for lw in self.layers:
            n += sum(w.nbytes for w in lw.linears()) + sum(t.numel() * t.element_size() for t in (lw.uk_t, lw.uv, lw.router) if t is not None)
            if lw.ff is not None:
                count = lw.ff.gate.count
                n += int(count * (1 - (1 - lw.top / count) ** rows) * sum(w.nbytes for w in lw.ff.linears()))
        return n


class DepthBuffers(LatentBuffers, ExpertBuffers):
    """Activations of up to `rows` rows, and their residuals at all depths."""

    def __init__(self, spec, weights, rows, direct, dtype, device):
        def buf(*shape, dtype=dtype):
            return torch.zeros(shape, dtype=dtype, device=device)
        mixers, layers, ld = [lay.mixer for lay in spec.layers], weights.layers, HK.pad8(spec.width)
        self.rows = rows
        # a depth more than there are: the average that goes on from the last layer (whole 16-byte pieces between the depths)
        self.history = buf(len(layers) + 2, (rows + 3) // 4 * 4, spec.width, dtype=F32)
        self.h, self.rounded = buf(rows, ld), buf(rows, ld)
        self.y = buf(rows, spec.width, dtype=F32)
        self.side = buf(len(layers), rows, weights.side.shape[2])
        self.side_act = buf(rows, weights.side.shape[2])
        self.proj = {n: buf(rows, n) for n in {lw.proj.n_main for lw in layers}}
        self.ctx = {n: buf(rows, n) for n in {m.out_channels for m in mixers}}
        self.convolved = {n: buf(rows, n) for n in {lw.conv.channels for lw in layers if lw.conv is not None}}
        memory = [m for m in mixers if m.kind == "ssd"]
        self.dt = buf(rows * max((m.heads for m in memory), default=0), dtype=F32)
        self.y_heads = buf(rows * max((m.out_channels for m in memory), default=0), dtype=F32)
        self.act = {lw.up.n_main: buf(rows, lw.up.n_main) for lw in layers if lw.up is not None}
        self.latent_buffers(buf, mixers, layers)
        self.expert_buffers(buf, spec, layers, direct, dtype, device)
        self.logits = {n: buf(rows, n, dtype=F32) for n in {lw.router.shape[0] for lw in layers if lw.router is not None}}
        channels = max([spec.width] + [w.N for lw in layers for w in lw.linears()])
        self.workspace = HK.linear_workspace(rows, channels, device) if rows > 16 else None


class DepthDecoder(HeadMixing, LatentMixing, StateSpaceMixing, ExpertMixing, HybridDecoder):
    # larger routers are multiplied beside the mixer's projections, with a launch for the choice (64 logits of 4096 features in the
    # norm's launch cost one row 10 us, the launch 4)
    router_bytes = 128 << 10

    def _rows_buffers(self, rows):
        size = rows if rows <= 16 else max(64, 1 << (rows - 1).bit_length())
        if size not in self._buffers:
            self._buffers[size] = DepthBuffers(self.spec, self.w, size, self._direct(size), self.dtype, self.dev)
        return self._buffers[size]

    def _projections(self, i, b, n):
        """What the mixer, a dense feed-forward and a router make of the normed rows.  Returns the mixer's, and the router's logits (None:
        the norm's launch has routed the rows)."""
        m, lw = self.spec.layers[i].mixer, self.w.layers[i]
        proj = b.proj[lw.proj.n_main]
        dt = b.dt[:n * m.heads] if m.kind == "ssd" else None
        calls = [(b.h, lw.proj, proj, dict(tail=dt, bias=lw.proj_bias, workspace=b.workspace))]
        if lw.up is not None:
            calls.append((b.h, lw.up, b.act[lw.up.n_main], dict(act=H.ACT_RELU_SQUARE, workspace=b.workspace)))
        logits = None
        if lw.router is not None and not self._routed_by_norm(i, b):
            logits = b.logits[lw.router_linear.n_main]
            calls.append((b.h, lw.router_linear, logits, dict(workspace=b.workspace)))
        HK.linear_group(n, *calls)
        return proj, dt, logits

    def _mixer(self, i, b, rows, proj, dt):
        """The heads' results, before the output projection."""
        m, lw = self.spec.layers[i].mixer, self.w.layers[i]
        if m.kind == "latent":
            return self._latent(i, lw, b, rows, proj, (proj, lw.proj.n_main - m.out_channels))
        if m.kind == "heads":
            return self._heads(i, lw, b, rows, proj)
        return self._state_space(i, lw, b, rows, proj, dt)

    def _layers(self, rows, pos_out=None):
        """All layers over the rows; h holds the model's norm of them."""
        spec, w, n = self.spec, self.w, rows.n
        b, depths = self._rows_buffers(n), len(spec.layers)
        self._lists_ahead(rows)

        def ahead(i):
            """the norm in front of layer i, and its routing"""
            if i == depths:
                return dict(norm_weight=w.final_norm)
            return dict(norm_weight=w.layers[i].norm, **(self._routed_by_norm(i, b) if isinstance(spec.layers[i].mlp, Experts) else {}))
        common = dict(rows=n, eps=spec.eps, h=b.h)
        HK.depth_norm(b.history, 0, table=w.embed, embed_scale=spec.embed_scale, ids=rows.ids, ids_index=rows.ids_index, pos_out=pos_out,
                      side_table=w.side, side=b.side, next=1, **ahead(0), **common)
        for i, layer in enumerate(spec.layers):
            lw, x = w.layers[i], b.history[i + 1]
            add = dict(ld=spec.width, accumulate=True, workspace=b.workspace)
            proj, dt, logits = self._projections(i, b, n)
            HK.linear(self._mixer(i, b, rows, proj, dt), lw.out, x, n, **add)
            parts = {}
            if isinstance(layer.mlp, Experts):
                parts = self._mixture(i, b, n, logits)
            elif layer.mlp is not None:
                HK.linear(b.act[lw.up.n_main], lw.down, x, n, **add)
            HK.add_parts(x, n, b.rounded, **parts)
            HK.linear(b.rounded, lw.side_gate, b.side_act, n, act=H.ACT_GELU_TANH, mul=b.side[i], workspace=b.workspace)
            HK.linear(b.side_act, lw.side_proj, b.y, n, ld=spec.width, workspace=b.workspace)
            going_on = i + 1 < depths or self.probe is not None
            HK.depth_norm(b.history, i + 2, weights=lw.average, y=b.y, y_weight=lw.side_norm, next=i + 2 if going_on else None,
                          **ahead(i + 1), **common)
            if self.probe is not None:
                self.probe(i, b.history[i + 2, :n].clone())
        return b, None

    def _logits(self, b, done, count, out, gather=None):
        h = b.h
        if gather is not None:
            if self._head_h is None:
                self._head_h = torch.zeros((self.head_rows, h.shape[1]), dtype=self.dtype, device=self.dev)
            h = self._head_h
            torch.index_select(b.h, 0, gather, out=h[:count])
        HK.linear(h, self.w.head, out, count, ld=self.spec.vocab, cap=self.spec.logit_cap)
