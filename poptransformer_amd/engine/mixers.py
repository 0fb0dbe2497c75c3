"""Mixers and mixtures of experts that the executors of several designs run, as mix-ins of HybridDecoder, with the row buffers each
of them needs: attention over latents, attention by heads, the state-space recurrence, experts.

What a mix-in reads: `spec`, `store`, `dtype`, `dev`, `_scratch` of the decoder; of the row buffers `b` what its buffers class makes,
`rows`, `workspace` and `ctx` (the heads' results by their number of channels); of the layer's weights `lw` the tensors of its
own mechanism.
"""
import numpy as np
import torch

from .. import _hybrid_lib as H
from .. import hybrid_kernels as HK
from .hybrid import F32, ClampedGLU, Experts


class Angles:
    def _cos_sin(self, rot, pairs=None):
        """Angles of all positions (None without a rotation); `pairs`: of so many pairs, the ones past the rotation's stay."""
        if rot is None:
            return None
        if not hasattr(self, "_angles"):
            self._angles = {}
        key = (*rot.numbers(), pairs)
        if key not in self._angles:
            self._angles[key] = torch.from_numpy(rot.angles(self.store.max_len, pairs)).to(self.dev)
        return self._angles[key]


# ------------------------------------------------------------------------------------------- latents
class LatentBuffers:
    def latent_buffers(self, buf, mixers, layers):
        """cq and q by their channels; `layers`: the layers' weights beside their mixers"""
        mine = [lw for m, lw in zip(mixers, layers) if m.kind == "latent"]
        self._buf, self._absorbed = buf, {}
        self.cq = {n: buf(self.rows, n) for n in {lw.uq.K for lw in mine}}
        self.q = {n: buf(self.rows, n) for n in {lw.uq.n_main for lw in mine}}

    def absorbed(self, heads, R, P, splits):
        """(queries against the latent, the parts' sums, their softmax states)"""
        key = (heads, R, P, splits)
        if key not in self._absorbed:
            n = self.rows * heads
            self._absorbed[key] = (self._buf(n, R + P), self._buf(n * splits, R, dtype=F32), self._buf(n * splits, 2, dtype=F32))
        return self._absorbed[key]


class LatentMixing(Angles):
    absorbed_rows = 16               # sequences with up to this many rows in a pass work on the cached rows themselves
    _key_lists = None

    def _latent_splits(self, rows, mixer):
        """Parts of the window per row: enough workgroups to fill the machine, at least 64 keys per part.  Fixed per shape, since
        the launch is replayed while the context grows."""
        wgs = rows * (-(-mixer.heads // 16) if self.dtype == torch.bfloat16 else mixer.heads)
        keys = min(mixer.window or self.store.max_len, self.store.max_len)
        return max(1, min(256 // wgs, -(-keys // 64), 64))

    def _keys(self, rows, window):
        """Cache rows that a pass's rows look at, sequence after sequence: (slots, positions), and where position 0 of a tile's
        sequence would lie among them.  One list per distinct window of a pass."""
        if self._key_lists is None or self._key_lists[0] is not rows:
            self._key_lists = (rows, {})
        lists = self._key_lists[1]
        if window not in lists:
            slots, places, zero, at = [], [], [], 0
            for slot, p0, count in rows.portions:
                first = max(0, p0 - window + 1) if window is not None else 0
                n = p0 + count - first
                slots.append(np.full(n, slot, np.int32))
                places.append(np.arange(first, first + n, dtype=np.int32))
                zero += [at - first] * -(-count // H.LATENT_TILE)
                at += n
            flat = torch.from_numpy(np.concatenate(slots + places + [np.array(zero, np.int32)])).to(self.dev)
            slot, pos, tile_key = torch.split(flat, [at, at, len(zero)])
            lists[window] = ((slot, pos), (*rows.tiles[:2], tile_key))
        return lists[window]

    def _takes_heads(self, i, rows):
        """Whether the pass makes keys and values of all heads for layer i (else it works on the cached rows themselves)."""
        return self.w.layers[i].kv is not None and not rows.single and rows.longest > self.absorbed_rows

    def _lists_ahead(self, rows):
        """Makes the key lists of a pass before its first launch: the copy to the device would wait for those ahead of it."""
        for i, lay in enumerate(self.spec.layers):
            if lay.mixer.kind == "latent" and self._takes_heads(i, rows):
                self._keys(rows, lay.mixer.window)

    def _latent(self, i, lw, b, rows, proj, gates):
        """The heads' gated results of layer i, before the output projection; gates: as LatentAttention takes them."""
        m, n = self.spec.layers[i].mixer, rows.n
        heads, D, P, E, R = m.sizes[:5]
        cq, q, ctx = b.cq[lw.uq.K], b.q[lw.uq.n_main], b.ctx[m.out_channels]
        ring, = self.store.stores[i if m.source is None else m.source]
        att = HK.LatentAttention(m.sizes, m.scale, m.window, self.spec.eps, lw.q_norm, lw.kv_norm, self._cos_sin(m.rot, P // 2), ring, n,
                                 rows.slot, rows.pos)
        att.append(proj, cq)
        HK.linear(cq, lw.uq, q, n, workspace=b.workspace)
        if not self._takes_heads(i, rows):
            splits = self._latent_splits(b.rows, m)
            q_latent, part_o, part_ml = b.absorbed(heads, R, P, splits)
            att.absorbed(q, lw.uk_t, q_latent, splits, part_o, part_ml, lw.uv, gates, ctx)
        else:
            keys, tiles = self._keys(rows, m.window)
            count = keys[0].numel()
            # latents, rotated parts, then keys and values of all heads
            sizes = [count * R, count * P, count * lw.kv.n_main]
            flat = self._scratch(2 * sum(sizes))[:2 * sum(sizes)].view(self.dtype)
            latent, rot, kv = torch.split(flat, sizes)
            att.over_heads(q, keys, latent.view(count, R), rot.view(count, P), lw.kv, kv.view(count, -1), tiles, gates, ctx)
        return ctx


# ------------------------------------------------------------------------------------------- heads
class HeadMixing(Angles):
    def _head_splits(self, rows, mixer):
        """Parts of the visible keys per (row, key head) of a decode pass, and the scratch they meet in.  Fixed per shape (the
        launch is replayed while the context grows): enough workgroups to fill the machine, at least 64 keys per part."""
        m = mixer
        key = (rows, m.heads, m.kv_heads, m.stored_dim, m.stored_vdim, m.maps, m.keep, m.span)
        if key not in self._splits_for:
            group, most = m.heads // m.kv_heads, 4 // m.maps
            wgs = rows * m.kv_heads * -(-group // (group if group <= 2 // m.maps else most))
            keys = min(m.keep + m.span, self.store.max_len)
            splits = max(1, min(768 // wgs, -(-keys // 64), 64)) if keys > 256 else 1
            self._splits_for[key] = (splits, HK.head_workspace(rows, m, splits, self.dev) if splits > 1 else None)
        return self._splits_for[key]

    def _heads(self, i, lw, b, rows, proj, gates=None):
        """The heads' results of layer i, before the output projection."""
        m, n = self.spec.layers[i].mixer, rows.n
        ctx, conv = b.ctx[m.out_channels], None
        if lw.conv is not None:
            conv = (lw.conv, self.store.recent[i])
            if not rows.single:
                raw, proj = proj, b.convolved[proj.shape[1]]
                lw.conv(raw, 0, proj, conv[1], n, rows.slot, rows.pos, rows.last, rows.tiles)
        att = HK.HeadAttention(m, self.spec.eps, lw.q_norm, lw.k_norm, self._cos_sin(m.rot), lw.sink, lw.lam, *self.store.stores[i], proj, n,
                               rows.slot, rows.pos, gates, ctx, lw.far)
        if rows.single:
            att.decode(*self._head_splits(n, m), conv)
        else:
            att.prompt(rows.tiles)
        return ctx


# ------------------------------------------------------------------------------------------- state space
class StateSpaceMixing:
    scanned_rows = 8                 # sequences with up to this many rows in a pass are worked through token by token

    def _state_space(self, i, lw, b, rows, proj, dt):
        """The heads' normed results of layer i, before the output projection.  proj rows hold z | x | b | c."""
        m, n = self.spec.layers[i].mixer, rows.n
        D, E, ring = m.stored_dim, m.stored_vdim, self.store.recent[i]
        y = b.y_heads[:n * m.out_channels].view(n, -1)
        x, x_at, conv = proj, m.out_channels, (lw.conv, ring)
        if not rows.single:
            x, x_at, conv = b.convolved[lw.conv.channels], 0, None
            lw.conv(proj, m.out_channels, x, ring, n, rows.slot, rows.pos, rows.last, rows.tiles)
        HK.ssd(x, x_at, n, m.heads, m.groups, D, E, dt, lw.ssd, self.store.stores[i][0], rows.slot, rows.seqs, rows.longest, y,
               rows.longest > self.scanned_rows, self._scratch, rows.pos, conv)
        ctx = b.ctx[m.out_channels]
        HK.gated_norm(y, proj, lw.head_norm, ctx, n, m.heads, E, m.vdim, m.norm_parts, self.spec.eps)
        return ctx


# ------------------------------------------------------------------------------------------- experts
def glu_pair(glu):
    """The epilogue between a feed-forward's gate / up pair and its down projection, as keywords of the products."""
    if isinstance(glu, ClampedGLU):
        return dict(pair=H.PAIR_CLAMPED, limit=glu.limit, slope=glu.slope)
    return dict(pair=H.PAIR_SWIGLU)


class ExpertBuffers:
    def expert_buffers(self, buf, spec, layers, direct, dtype, device):
        """Routing, activations and results of the layers' mixtures (`act` of whole feed-forwards is there already)"""
        rows = self.rows
        self.parts, self.routing, self.lists, self.logits = {}, {}, {}, {}
        for lay, lw in zip(spec.layers, layers):
            e = lay.mlp
            if not isinstance(e, Experts):
                continue
            choices = e.top + (e.shared is not None)
            if e.routing_key not in self.routing:
                self.routing[e.routing_key] = HK.Routing(rows, e.count, e.top, e.shared is not None, e.scale, device,
                                                         H.SCORE_SIGMOID if e.score == "sigmoid" else H.SCORE_SOFTMAX, e.groups, e.keep, e.share)
            n = lw.ff.gate.n_main
            if lw.shared is not None:
                self.act[lw.shared.gate.n_main] = buf(rows, lw.shared.gate.n_main)
                n = max(n, lw.shared.gate.n_main) if direct else n
            if (choices, n) not in self.act:
                self.act[choices, n] = buf(rows * choices, n)
            if choices not in self.parts:
                self.parts[choices] = buf(rows * choices, spec.width, dtype=F32 if direct else dtype)
            if dtype == F32:
                self.logits[lw.router.shape[0]] = buf(rows, lw.router.shape[0], dtype=F32)
            if not direct:
                for t in (128, 256):
                    self.lists[e.count, e.top, t] = HK.expert_lists(rows, e.top, e.count, t, device)


class ExpertMixing:
    direct_rows = 16                 # passes of up to this many bf16 rows find their experts' rows without lists
    # routers up to this size are multiplied in the norm's launch by passes of up to so many rows (every row reads all of it: 2048
    # rows of 4096 features and 33 logits take 43 us that way, 19 + 21 with a launch for the routing, 512 rows 16 against 10 + 15)
    router_bytes, router_rows = 1 << 20, 512
    tall_rows = 128                  # rows per expert, on average, above which their lists are cut into tiles of 256 (else 128)

    def _direct(self, rows):
        return self.dtype == torch.bfloat16 and rows <= self.direct_rows

    def _routing(self, i, b):
        return b.routing[self.spec.layers[i].mlp.routing_key]

    def _routed_by_norm(self, i, b):
        """What the norm's launch needs to route the rows to layer i's experts, where it does."""
        lw = self.w.layers[i]
        if lw.router is None or b.rows > self.router_rows or lw.router.numel() * lw.router.element_size() > self.router_bytes:
            return {}
        out = dict(router=lw.router, routing=self._routing(i, b))
        return out if lw.correction is None else dict(out, correction=lw.correction)

    def _mixture(self, i, b, n, logits=None):
        """The results of layer i's experts over the rows of b.h, as arguments of what adds them up; logits: the router's, where they
        are there already."""
        mlp, lw = self.spec.layers[i].mlp, self.w.layers[i]
        r = self._routing(i, b)
        if logits is not None:
            r(logits, n, lw.correction)
        elif not self._routed_by_norm(i, b):
            if self.dtype == torch.bfloat16:
                r.by_product(b.h, lw.router_linear, n, lw.correction)
            else:
                logits = b.logits[lw.router.shape[0]]
                HK.linear(b.h, lw.router_linear, logits, n)
                r(logits, n, lw.correction)
        parts = b.parts[r.choices]
        result = dict(parts=parts, parts_ld=r.choices, part_weight=r.weights)
        pair, down = dict(w=lw.ff.gate, up=lw.ff.up, **glu_pair(mlp.expert)), dict(w=lw.ff.down)
        if self._direct(b.rows):
            shared_pair = shared_down = None
            act_ld = lw.ff.gate.n_main
            if mlp.shared is not None:
                shared_pair, shared_down = dict(w=lw.shared.gate, up=lw.shared.up, **glu_pair(mlp.shared)), dict(w=lw.shared.down)
                act_ld = max(act_ld, lw.shared.gate.n_main)
            act = b.act[r.choices, act_ld]
            HK.experts(b.h, r, n, pair, act, shared_pair)
            HK.experts(act, r, n, down, parts, shared_down)
            return dict(result, n_parts=r.choices)
        tile = 256 if n * mlp.top > self.tall_rows * mlp.count else 128
        lists, act = b.lists[mlp.count, mlp.top, tile], b.act[r.choices, lw.ff.gate.n_main]
        HK.group_experts(r, n, tile, lists)
        HK.experts(b.h, r, n, pair, act, lists=lists, tile_rows=tile)
        HK.experts(act, r, n, down, parts, lists=lists, tile_rows=tile)
        result.update(n_parts=mlp.top)
        if mlp.shared is not None:
            self._dense(b, n, lw.shared, **glu_pair(mlp.shared))
            result.update(y=b.y, y_weight=(r.weights, mlp.top))
        return result

    def _dense(self, b, n, ff, **pair):
        act = b.act[ff.gate.n_main]
        HK.linear(b.h, ff.gate, act, n, up=ff.up, **pair)
        HK.linear(act, ff.down, b.y, n, ld=self.spec.width, workspace=b.workspace)
