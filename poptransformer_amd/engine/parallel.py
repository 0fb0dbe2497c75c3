"""Executor of decoders whose layers run mixer and feed-forward side by side on one fp32 residual:

    x <- x + gate1 * mixer(shift(n1(x))) + gate2 * ff(n2(x)),    gate = sigmoid(W n(x) + b)

with a norm in groups, a token shift in front of the mixer and latent attention.  Rows, sequences, sampling and the decode
loop are HybridDecoder's.

Launches of a layer in a decode iteration: norms and token shift; both residual gates with the mixer's down-projections;
latent norms and cache entry; queries; queries against the latent; attention over the cached rows; values; output projection
(its epilogue gates and adds to the residual); gate / up pair; down projection (likewise).  Prompts take keys and values of
every head instead of the middle three.
"""
from dataclasses import dataclass
from typing import List, Optional

import torch

from .. import _hybrid_lib as H
from .. import hybrid_kernels as HK
from .hybrid import F32, HybridDecoder
from .mixers import LatentBuffers, LatentMixing


@dataclass
class ParallelLayerWeights:
    norm1: torch.Tensor
    shift: torch.Tensor
    gate1: HK.WideWeight
    gate1_bias: torch.Tensor
    proj: HK.WideWeight              # query latent | cache entry (layers with a cache of their own), tail: the heads' gates
    q_norm: torch.Tensor
    kv_norm: Optional[torch.Tensor]
    uq: HK.WideWeight
    uk_t: torch.Tensor               # [heads, R, D]
    uv: torch.Tensor                 # [heads, E, R]
    kv: Optional[HK.WideWeight]      # keys of all heads | values of all heads, from the latent (None: the sizes are taken absorbed)
    out: HK.WideWeight
    norm2: Optional[torch.Tensor] = None
    gate2: Optional[HK.WideWeight] = None
    gate2_bias: Optional[torch.Tensor] = None
    gate: Optional[HK.WideWeight] = None
    gate_bias: Optional[torch.Tensor] = None
    up: Optional[HK.WideWeight] = None
    up_bias: Optional[torch.Tensor] = None
    down: Optional[HK.WideWeight] = None
    down_bias: Optional[torch.Tensor] = None

    def linears(self):
        """Every weight once, as a decode iteration reads them."""
        return [w for w in (self.gate1, self.proj, self.uq, self.out, self.gate2, self.gate, self.up, self.down) if w is not None]

    def feed_forward_bytes(self):
        return sum(w.nbytes for w in (self.gate2, self.gate, self.up, self.down))


@dataclass
class ParallelWeights:
    embed: torch.Tensor
    pos: torch.Tensor
    layers: List[ParallelLayerWeights]
    final_norm: torch.Tensor
    head: HK.WideWeight

    def nbytes(self):
        """Bytes of the weights, each counted once."""
        return self.head.nbytes + sum(sum(w.nbytes for w in lay.linears()) + sum(t.numel() * t.element_size() for t in (lay.uk_t, lay.uv))
                                      for lay in self.layers)


class ParallelBuffers(LatentBuffers):
    """Activations of up to `rows` rows."""

    def __init__(self, spec, weights, rows, dtype, device):
        def buf(*shape, dtype=dtype):
            return torch.zeros(shape, dtype=dtype, device=device)
        mixers, ld = [lay.mixer for lay in spec.layers], HK.pad8(spec.width)
        self.rows = rows
        self.x = buf(rows, spec.width, dtype=F32)
        self.h1, self.h2, self.hm = buf(rows, ld), buf(rows, ld), buf(rows, ld)
        self.gate1, self.gate2 = buf(rows, spec.width), buf(rows, spec.width)
        self.proj = {n: buf(rows, n) for n in {lw.proj.n_main for lw in weights.layers}}
        self.head_gates = {n: buf(rows, n, dtype=F32) for n in {m.heads for m in mixers}}
        self.latent_buffers(buf, mixers, weights.layers)
        self.ctx = {n: buf(rows, n) for n in {m.out_channels for m in mixers}}
        self.act = {n: buf(rows, n) for n in {lw.gate.n_main for lw in weights.layers if lw.gate is not None}}
        channels = max(w.N for lw in weights.layers for w in lw.linears())
        self.workspace = HK.linear_workspace(rows, channels, device) if rows > 16 else None


class ParallelDecoder(LatentMixing, HybridDecoder):
    # passes of up to branch_rows single rows run a feed-forward of at least branch_bytes on a stream beside the mixer: what two
    # streams cost to part and meet (measured: feed-forwards of 80 MB lose 4 us per layer by it, of 300 MB gain 11)
    branch_rows = 16
    branch_bytes = 128 << 20

    def __init__(self, spec, weights, device="cuda", slots=None):
        super().__init__(spec, weights, device, slots)
        self._side = torch.cuda.Stream()

    def _rows_buffers(self, rows):
        size = rows if rows <= 16 else max(64, 1 << (rows - 1).bit_length())
        if size not in self._buffers:
            self._buffers[size] = ParallelBuffers(self.spec, self.w, size, self.dtype, self.dev)
        return self._buffers[size]

    def _mixer(self, i, b, rows):
        """The heads' gated results, before the output projection."""
        lw = self.w.layers[i]
        return self._latent(i, lw, b, rows, b.proj[lw.proj.n_main], b.head_gates[self.spec.layers[i].mixer.heads])

    def _projections(self, i, b, n, mixer=True, ff=True):
        """The sublayers' residual gates, and the mixer's down-projections."""
        lw, ld, calls = self.w.layers[i], self.spec.width, []
        if mixer:
            calls += [(b.h1, lw.gate1, b.gate1, dict(ld=ld, bias=lw.gate1_bias, act=H.ACT_SIGMOID, workspace=b.workspace)),
                      (b.hm, lw.proj, b.proj[lw.proj.n_main], dict(tail=b.head_gates[self.spec.layers[i].mixer.heads], workspace=b.workspace))]
        if ff:
            calls.append((b.h2, lw.gate2, b.gate2, dict(ld=ld, bias=lw.gate2_bias, act=H.ACT_SIGMOID, workspace=b.workspace)))
        HK.linear_group(n, *calls)

    def _output(self, i, b, n, ctx):
        """x += gate1 * (W_o ctx)"""
        HK.linear(ctx, self.w.layers[i].out, b.x, n, ld=self.spec.width, mul=b.gate1, accumulate=True, workspace=b.workspace)

    def _feed_forward(self, i, b, rows):
        lw, n = self.w.layers[i], rows.n
        act = b.act[lw.gate.n_main]
        HK.linear(b.h2, lw.gate, act, n, up=lw.up, pair=H.PAIR_SWIGLU, bias=lw.gate_bias, bias2=lw.up_bias)
        HK.linear(act, lw.down, b.x, n, ld=self.spec.width, bias=lw.down_bias, mul=b.gate2, accumulate=True, workspace=b.workspace)

    def _layers(self, rows, pos_out=None):
        """All layers over the rows; the residual is left in the buffers."""
        spec, w, store, n = self.spec, self.w, self.store, rows.n
        b = self._rows_buffers(n)
        last = None if rows.single else rows.last
        self._lists_ahead(rows)
        for i, layer in enumerate(spec.layers):
            lw, ff = w.layers[i], layer.mlp is not None
            first = dict(table=w.embed, pos_table=w.pos, embed_scale=spec.embed_scale, ids=rows.ids, ids_index=rows.ids_index,
                         pos_out=pos_out) if i == 0 else {}
            HK.shift_norm(b.x, n, spec.norm_groups, spec.eps, lw.norm1, b.h1, lw.norm2, b.h2 if ff else None, lw.shift, b.hm,
                          store.shifted[i], rows.slot, last, rows.pos, store.max_len, **first)
            if ff and rows.single and n <= self.branch_rows and lw.feed_forward_bytes() >= self.branch_bytes:
                # the feed-forward is bound by its weights, the mixer by a chain of short launches; they meet in the residual
                main = torch.cuda.current_stream()
                self._side.wait_stream(main)
                with torch.cuda.stream(self._side):
                    self._projections(i, b, n, mixer=False)
                    self._feed_forward(i, b, rows)
                self._projections(i, b, n, ff=False)
                ctx = self._mixer(i, b, rows)
                main.wait_stream(self._side)
                self._output(i, b, n, ctx)
            else:
                self._projections(i, b, n, ff=ff)
                self._output(i, b, n, self._mixer(i, b, rows))
                if ff:
                    self._feed_forward(i, b, rows)
            if self.probe is not None:
                self.probe(i, b.x[:n].clone())
        return b, None

    def _logits(self, b, done, count, out, gather=None):
        spec, h = self.spec, b.h1
        if gather is not None:
            if self._head_h is None:
                self._head_h = torch.zeros((self.head_rows, h.shape[1]), dtype=self.dtype, device=self.dev)
            h = self._head_h
        HK.shift_norm(b.x, count, spec.norm_groups, spec.eps, self.w.final_norm, h, gather=gather)
        HK.linear(h, self.w.head, out, count, ld=spec.vocab)
