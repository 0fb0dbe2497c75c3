"""The host side of the decode loop (models/base_model.py:271-355) that the executors share: how many leading
iterations only read the prompt, the recording of one iteration into a HIP graph, and the loop itself.

An executor provides `spec` (batch, max_len, pad_id, eos_id, early_stop), `reset(input_ids)`, `step_fn()` (one iteration
from device state only) and the device tensors `container`, `step`, `keep_going`; optionally `consume_prompt(n)`.
"""
import numpy as np
import torch


class DecodeLoop:
    graph = None

    def checked_ids(self, input_ids):
        """input_ids as a host tensor of the container's shape; kept for `prompt_positions`."""
        s = self.spec
        ids = torch.as_tensor(np.asarray(input_ids, np.int32))
        if tuple(ids.shape) != (s.batch, s.max_len):
            raise ValueError(f"input_ids must be [{s.batch}, {s.max_len}], got {tuple(ids.shape)}")
        self._host_ids = ids.numpy().copy()
        return ids

    def prompt_positions(self):
        """How many leading loop iterations only read the prompt: their `next_ids` are dropped because the
        container already holds a token at the next position (models/base_model.py:313-318), and no
        sequence meets its end token there.  These are the positions `consume_prompt` may take at once."""
        s, ids = self.spec, self._host_ids
        n = s.max_len - 1
        for row in ids:
            later = row[1:]
            pads = np.nonzero(later == s.pad_id)[0]
            ends = np.nonzero(later == s.eos_id)[0]
            n = min(n, int(pads[0]) if len(pads) else s.max_len - 1, int(ends[0]) if len(ends) else s.max_len - 1)
        return max(n, 0)

    def checked_prompt_count(self, n):
        """The argument of `consume_prompt`, checked; None: all prompt positions."""
        limit = self.prompt_positions()
        n = limit if n is None else int(n)
        if n < 0 or n > limit:
            raise ValueError(f"consume_prompt: n = {n} outside [0, {limit}] (the prompt's own positions before any end token)")
        if int(self.step.item()) != 0:
            raise RuntimeError("consume_prompt must follow reset()")
        return n

    def capture(self):
        """Record one loop iteration into a HIP graph (after an eager iteration has warmed up
        every code path).  The iteration depends on device state only, so it can be replayed."""
        self.reset(np.zeros((self.spec.batch, self.spec.max_len), np.int32))
        torch.cuda.synchronize()         # the stream of the recording does not wait for what prepared the buffers
        with torch.cuda.stream(self._stream):
            self.step_fn()
            torch.cuda.synchronize()
            self.graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(self.graph, stream=self._stream):
                self.step_fn()
        torch.cuda.synchronize()
        return self.graph

    def run_steps(self, n):
        if self.graph is None:
            for _ in range(n):
                self.step_fn()
        else:
            for _ in range(n):
                self.graph.replay()

    def check_finished(self):
        """Hook: raise when the iterations that have just been synchronised reported a failure."""

    def run(self, input_ids, max_loop, check_every=16, prompt_passes=False):
        """The whole generation (one `session.run` of the reference, poptransformer/sessions.py:47-49).
        Returns (container, step) like the anchors 'Loop:0' and 'Loop:1'.  prompt_passes: the leading
        iterations that only read the prompt run as passes over several positions, where the executor has them."""
        self.reset(input_ids)
        done = 0
        if prompt_passes and hasattr(self, "consume_prompt"):
            n = min(self.prompt_positions(), max_loop)
            if n > 0:
                done = self.consume_prompt(n)
        while done < max_loop:
            n = min(check_every, max_loop - done) if self.spec.early_stop else max_loop - done
            self.run_steps(n)
            done += n
            if self.spec.early_stop and int(self.keep_going.item()) == 0:
                break
        torch.cuda.synchronize()
        self.check_finished()
        return self.container.cpu().numpy(), int(self.step.item())
