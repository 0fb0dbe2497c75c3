"""Executor of decoders whose fp32 residual takes the norms of its sublayers' results,

    x <- x + norm1(mixer(x)),    x <- x + norm2(ff(x)),

with attention by heads and feed-forwards that may be mixtures of experts.  The sublayers read x itself.  Rows, sequences,
sampling and the decode loop are HybridDecoder's.

Launches of a layer in a decode iteration: projections; attention (norms, rotation and cache entry with it, the parts of the
visible keys merged by a second launch); output projection; result norm, which also routes the row; gate / up pair and down
projection of the chosen experts and the shared one (or of the dense feed-forward); result norm.  Passes of many rows work
through the experts' lists of rows, and route in a launch of its own.
"""
from dataclasses import dataclass
from typing import List, Optional

import torch

from .. import hybrid_kernels as HK
from .hybrid import F32, Experts, HybridDecoder
from .mixers import ExpertBuffers, ExpertMixing, HeadMixing, glu_pair


@dataclass
class FeedForwardWeights:
    """Gate, up and down of a feed-forward, or of every expert of a mixture."""
    gate: object                     # WideWeight, or ExpertWeight
    up: object
    down: object

    def linears(self):
        return [self.gate, self.up, self.down]


@dataclass
class ResultNormLayerWeights:
    norm1: torch.Tensor
    proj: HK.WideWeight              # q | k | v (none where the values are the keys) | gate per feature, tail: gates per head
    proj_bias: Optional[torch.Tensor]
    out: HK.WideWeight
    q_norm: torch.Tensor
    k_norm: torch.Tensor
    sink: Optional[torch.Tensor] = None
    lam: float = 0.0                 # weight of the second map
    far: Optional[tuple] = None      # (far1, far2) of the heads' distance penalty
    conv: Optional[HK.ShortConv] = None
    norm2: Optional[torch.Tensor] = None
    ff: Optional[FeedForwardWeights] = None          # dense, or the routed experts
    shared: Optional[FeedForwardWeights] = None
    router: Optional[torch.Tensor] = None            # [experts (+ the shared one's gate), padded width]
    router_linear: Optional[HK.WideWeight] = None    # the same as a Linear
    top: int = 0
    correction: Optional[torch.Tensor] = None        # of the router's scores

    def active_parameters(self):
        """Parameters of the products that one row goes through."""
        parts = [(w, 1) for w in (self.proj, self.out)] + [(w, max(self.top, 1)) for w in (self.ff.linears() if self.ff else ())]
        parts += [(w, 1) for w in (self.shared.linears() if self.shared else ())]
        return sum(w.n_main * w.K * times for w, times in parts)


@dataclass
class ResultNormWeights:
    embed: torch.Tensor
    layers: List[ResultNormLayerWeights]
    final_norm: torch.Tensor
    head: HK.WideWeight

    def nbytes(self, rows=1):
        """Bytes of the weights that a pass of `rows` rows reads: of a mixture the experts that so many choose on average, where every
        choice is as likely as another."""
        n = self.head.nbytes
        for lw in self.layers:
            n += lw.proj.nbytes + lw.out.nbytes
            for part in (lw.ff, lw.shared):
                if part is not None:
                    n += sum(w.nbytes for w in part.linears())
            if lw.router is not None:
                n += lw.router.numel() * lw.router.element_size()
                count = lw.ff.gate.count
                n += int((count * (1 - (1 - lw.top / count) ** rows) - 1) * sum(w.nbytes for w in lw.ff.linears()))
        return n


class ResultNormBuffers(ExpertBuffers):
    """Activations of up to `rows` rows."""

    def __init__(self, spec, weights, rows, direct, dtype, device):
        def buf(*shape, dtype=dtype):
            return torch.zeros(shape, dtype=dtype, device=device)
        self.rows = rows
        self.x = buf(rows, spec.width, dtype=F32)
        self.h = buf(rows, HK.pad8(spec.width))
        self.y = buf(rows, spec.width, dtype=F32)
        self.proj = {n: buf(rows, n) for n in {lw.proj.n_main for lw in weights.layers}}
        self.head_gates = {n: buf(rows, n, dtype=F32) for n in {lw.proj.tail for lw in weights.layers} if n}
        self.ctx = {n: buf(rows, n) for n in {lay.mixer.out_channels for lay in spec.layers}}
        self.act = {lw.ff.gate.n_main: buf(rows, lw.ff.gate.n_main) for lay, lw in zip(spec.layers, weights.layers)
                    if lay.mlp is not None and not isinstance(lay.mlp, Experts)}
        self.expert_buffers(buf, spec, weights.layers, direct, dtype, device)
        channels = max([spec.width] + [lw.proj.N for lw in weights.layers])
        self.workspace = HK.linear_workspace(rows, channels, device) if rows > 16 else None


class ResultNormDecoder(HeadMixing, ExpertMixing, HybridDecoder):
    def _rows_buffers(self, rows):
        size = rows if rows <= 16 else max(64, 1 << (rows - 1).bit_length())
        if size not in self._buffers:
            self._buffers[size] = ResultNormBuffers(self.spec, self.w, size, self._direct(size), self.dtype, self.dev)
        return self._buffers[size]

    def _mixer(self, i, b, rows):
        lw, n = self.w.layers[i], rows.n
        proj, gates = b.proj[lw.proj.n_main], b.head_gates[lw.proj.tail] if lw.proj.tail else None
        HK.linear(b.h, lw.proj, proj, n, tail=gates, bias=lw.proj_bias, workspace=b.workspace)
        HK.linear(self._heads(i, lw, b, rows, proj, gates), lw.out, b.y, n, ld=self.spec.width, workspace=b.workspace)

    def _feed_forward(self, i, b, n):
        """The feed-forward's result, as arguments of result_norm."""
        mlp = self.spec.layers[i].mlp
        if isinstance(mlp, Experts):
            return self._mixture(i, b, n)
        self._dense(b, n, self.w.layers[i].ff, **glu_pair(mlp))
        return dict(y=b.y)

    def _layers(self, rows, pos_out=None):
        """All layers over the rows; h holds the model's norm of them."""
        spec, w, n = self.spec, self.w, rows.n
        b = self._rows_buffers(n)
        common = dict(x=b.x, rows=n, eps=spec.eps, h=b.h)
        HK.result_norm(table=w.embed, embed_scale=spec.embed_scale, ids=rows.ids, ids_index=rows.ids_index, pos_out=pos_out, **common)
        for i, layer in enumerate(spec.layers):
            lw, ff = w.layers[i], layer.mlp is not None
            last = dict(final_weight=w.final_norm) if i == len(spec.layers) - 1 else {}
            self._mixer(i, b, rows)
            HK.result_norm(y=b.y, weight=lw.norm1, **(self._routed_by_norm(i, b) if ff else last), **common)
            if ff:
                HK.result_norm(weight=lw.norm2, **self._feed_forward(i, b, n), **last, **common)
            if self.probe is not None:
                self.probe(i, b.x[:n].clone())
        return b, None

    def _logits(self, b, done, count, out, gather=None):
        h = b.h
        if gather is not None:
            if self._head_h is None:
                self._head_h = torch.zeros((self.head_rows, h.shape[1]), dtype=self.dtype, device=self.dev)
            h = self._head_h
            torch.index_select(b.h, 0, gather, out=h[:count])
        HK.linear(h, self.w.head, out, count, ld=self.spec.vocab)
