"""Cache and state of the sequences a hybrid decoder works on.

A sequence holds one SLOT while it lives.  Per layer run (a layer whose weights are another layer's has a cache of its
own) a slot is
  * for windowed attention: a ring of key rows, position p in row p % ring_len, and one fp32 factor per position;
  * for matrix memory: the fp32 state, zero before the first token.
Ring rows need no clearing: a position is only looked at once its own sequence has written it.
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
        self.length = []                      # tokens each slot holds, -1: free
        self._grow(slots)

    def ring_len(self, mixer):
        n = self.max_len if mixer.window is None else min(self.max_len, mixer.window - 1 + self.portion)
        return (n + 63) // 64 * 64

    def _grow(self, slots):
        for i, layer in enumerate(self.spec.layers):
            m = layer.mixer
            if m.kind == "attention":
                n = self.ring_len(m)
                new = (torch.zeros((slots, m.kv_heads, n, HK.pad8(m.dim)), dtype=self.dtype, device=self.dev),
                       torch.zeros((slots, n), dtype=torch.float32, device=self.dev))
            else:
                new = (HK.mlstm_state(slots, m.heads, m.dim, m.vdim, self.dev),)
            for old, t in zip(self.stores[i] or (), new):
                t[:old.shape[0]].copy_(old)
            self.stores[i] = new
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
            if layer.mixer.kind == "mlstm":
                for slot in slots:
                    store[0][slot].zero_()
        for slot in slots:
            self.length[slot] = 0

    @property
    def nbytes(self):
        return sum(t.numel() * t.element_size() for store in self.stores for t in store)
