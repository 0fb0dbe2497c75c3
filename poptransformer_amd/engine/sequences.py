"""Cache and state of the sequences a hybrid decoder works on.

A sequence holds one SLOT while it lives.  Per layer run (a layer whose weights are another layer's has a cache of its
own) a slot is
  * for windowed attention: a ring of key rows, position p in row p % ring_len, and one fp32 factor per position;
  * for attention by heads: rings of keys (normed, rotated) and values, the first `keep` positions in rows of their own before
    the ring of the others;
  * for latent attention: a ring of latents with their rotated key part - a layer that reads another one's cache has none;
  * for matrix memory and the state-space recurrence: the fp32 state, zero before the first token;
  * for a short convolution: a ring of its newest rows as they were projected;
and with a token shift per layer the normed fp32 row of the newest token.
Ring rows need no clearing: a position is only looked at once its own sequence has written it; nor does the shift's row,
which position 0 does not look at.
"""
import torch

from .. import hybrid_kernels as HK


class SequenceStore:
    def __init__(self, spec, dtype, slots, max_len, pass_rows, device="cuda"):
        """max_len: positions a sequence may reach.  pass_rows: most rows of one sequence in one pass (a windowed ring
        keeps that many rows beyond its window, so that a pass can append all of its keys before the first row looks)."""
        self.spec, self.dtype, self.dev = spec, dtype, device
        self.max_len = max_len
        self.portion = min(pass_rows, max_len)
        self.capacity = 0
        self.stores = [None] * len(spec.layers)
        self.shifted = [None] * len(spec.layers)      # fp32 [slots, width] per layer with a token shift
        self.recent = [None] * len(spec.layers)       # [slots, taps, channels] per layer with a short convolution
        self.length = []                      # tokens each slot holds, -1: free
        self._grow(slots)

    def cache_window(self, i):
        """The widest window over the cache of layer i: its own, and those of the layers that read it (None: everything)."""
        windows = [m.window for j, m in enumerate(lay.mixer for lay in self.spec.layers)
                   if j == i or getattr(m, "source", None) == i]
        return None if None in windows else max(windows)

    def ring_len(self, i):
        m = self.spec.layers[i].mixer
        if m.kind == "heads":
            n = max(min(self.max_len, m.keep + m.span - 1 + self.portion), m.keep + 1)
            return (n + 63) // 64 * 64
        window = self.cache_window(i)
        n = self.max_len if window is None else min(self.max_len, window - 1 + self.portion)
        return (n + 63) // 64 * 64

    def _grow(self, slots):
        def zeros(*shape, dtype=self.dtype):
            return torch.zeros(shape, dtype=dtype, device=self.dev)

        def moved(old, new):
            for o, t in zip(old or (), new):
                t[:o.shape[0]].copy_(o)
            return new
        for i, layer in enumerate(self.spec.layers):
            m = layer.mixer
            if m.kind == "attention":
                n = self.ring_len(i)
                new = (zeros(slots, m.kv_heads, n, HK.pad8(m.dim)), zeros(slots, n, dtype=torch.float32))
            elif m.kind == "heads":
                n = self.ring_len(i)
                new = (zeros(slots, m.kv_heads, m.maps, n, m.stored_dim), zeros(slots, m.kv_heads, n, m.stored_vdim))
            elif m.kind == "latent":
                new = (zeros(slots, self.ring_len(i), m.cache_row),) if m.source is None else ()
            elif m.kind == "ssd":
                new = (HK.ssd_state(slots, m.heads, m.stored_dim, m.stored_vdim, self.dev),)
            else:
                new = (HK.mlstm_state(slots, m.heads, m.dim, m.vdim, self.dev),)
            self.stores[i] = moved(self.stores[i], new)
            if getattr(m, "taps", 0):
                old = self.recent[i]
                self.recent[i], = moved(old if old is None else (old,), (zeros(slots, m.taps, m.conv_channels),))
            if layer.shift:
                old = self.shifted[i]
                self.shifted[i], = moved(old if old is None else (old,), (zeros(slots, self.spec.width, dtype=torch.float32),))
        self.length += [-1] * (slots - self.capacity)
        self.capacity = slots

    def open(self):
        """A slot for a new sequence, its recurrent state at the start; the store grows when all are taken."""
        if -1 not in self.length:
            self._grow(2 * self.capacity)
        slot = self.length.index(-1)
        self.restart([slot])
        return slot

    def close(self, slot):
        if self.length[slot] < 0:
            raise ValueError(f"slot {slot} is not in use")
        self.length[slot] = -1

    def restart(self, slots):
        """The given slots hold a sequence without tokens."""
        for layer, store in zip(self.spec.layers, self.stores):
            if layer.mixer.kind in ("mlstm", "ssd"):
                for slot in slots:
                    store[0][slot].zero_()
        for slot in slots:
            self.length[slot] = 0

    @property
    def nbytes(self):
        rest = [[t] for t in self.shifted + self.recent if t is not None]
        return sum(t.numel() * t.element_size() for store in self.stores + rest for t in store)
