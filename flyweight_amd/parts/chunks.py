"""Which rows of a step a recurrence walks in chunks side by side: the chunks of every long segment.

A recurrence whose step combines (a chunk's effect on the state is one decay and one sum) walks a prompt's rows in
chunks of ``CHUNK_ROWS`` at once: each chunk from a zero state, then the states ahead of the chunks, then the read-outs.
Segments of up to ``LONG_ROWS`` rows are walked in order."""

from __future__ import annotations

from typing import Dict

import numpy as np

from ..kernels import ops


class RecurrenceChunks:
    """For a mixer: asks the step's upload for the chunks (``Part.step_arrays``); mixers share one set."""

    CHUNK_ROWS = ops.DECAY_CHUNK
    LONG_ROWS = 32

    def step_arrays_key(self):
        return ("recurrence_chunks", self.CHUNK_ROWS, self.LONG_ROWS)

    def step_arrays(self, batch) -> Dict[str, np.ndarray]:
        if batch.all_decode:            # every segment one row: there is nothing to cut
            return {}
        row0 = np.asarray(batch.host_seg_row0, dtype=np.int64)
        lengths = row0[1:] - row0[:-1]
        counts = np.where(lengths > self.LONG_ROWS, -(-lengths // self.CHUNK_ROWS), 0)
        begins = np.concatenate([[0], np.cumsum(counts)])
        seg = np.repeat(np.arange(len(lengths)), counts)
        within = np.arange(int(begins[-1])) - np.repeat(begins[:-1], counts)
        return {"chunk_seg": seg.astype(np.int32), "chunk_row0": (row0[:-1][seg] + within * self.CHUNK_ROWS).astype(np.int32),
                "seg_chunk0": begins.astype(np.int32)}

    def chunk_arguments(self, ctx) -> dict:
        """What the recurrence's launch is told: the chunks (none in a step of single rows) and from which length on."""
        own = ctx.step_arrays(self) if not ctx.all_decode else {}
        if not own or own["chunk_seg"].numel() == 0:
            return {}
        lengths = np.diff(ctx.host_seg_row0)
        return {"chunks": (own["chunk_seg"], own["chunk_row0"], own["seg_chunk0"], self.LONG_ROWS, bool(lengths.min() > self.LONG_ROWS))}
