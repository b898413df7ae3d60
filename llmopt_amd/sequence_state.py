"""Per-sequence state in device memory: key / value rings, convolution rings, recurrent states.

A `StatePool` has a fixed number of slots; a live sequence owns one.  Everything a layer carries from
token to token is a region [slot][...] of one buffer per layer and kind, so kernels find a sequence's
part from the slot number alone (the second step word).  Slots need no clearing: a sequence starts at
position 0, where the kernels take state and history as zero, and rings only hand out rows that the
sequence itself has written.

A key / value ring keeps `capacity` positions per head (position p in row p % capacity).  Attention over
chunks or a sliding window needs one of them; attention over the whole sequence needs the longest context the
pool is made for.
"""
from __future__ import annotations

from dataclasses import dataclass

from .native import Runtime


class StateError(RuntimeError):
    """No free slot, or a sequence beyond what the pool holds."""


@dataclass(frozen=True)
class RingShape:
    """Keys and values of one attention layer."""
    kv_heads: int
    dim: int
    vdim: int
    span: int      # chunk or window; 0: the whole sequence
    capacity: int

    @staticmethod
    def of(kv_heads: int, dim: int, vdim: int, span: int, max_context: int) -> "RingShape":
        # positions below max_context never leave the first chunk or window when that is at least as long
        if span == 0 or span >= max_context:
            return RingShape(kv_heads, dim, vdim, 0, max_context)
        return RingShape(kv_heads, dim, vdim, span, span)


@dataclass(frozen=True)
class RecurrentShape:
    """Convolution inputs and state (state x vdim values per head) of one recurrent layer."""
    heads: int
    vdim: int
    state: int
    channels: int
    taps: int


@dataclass
class Sequence:
    slot: int
    position: int = 0  # tokens processed so far


class StatePool:
    def __init__(self, runtime: Runtime, shapes, slots: int, max_context: int, element_bytes: int):
        if slots < 1 or max_context < 1:
            raise StateError("a state pool needs at least one slot and one token of context")
        self.slots, self.max_context = slots, max_context
        self._free = list(range(slots))[::-1]
        self._live: set[int] = set()
        self.bytes = 0
        # per layer, for each of its shapes: (keys, values) or (convolution ring, state)
        self.regions = [tuple(self._region(runtime, shape, element_bytes) for shape in layer) for layer in shapes]

    def _region(self, runtime: Runtime, shape, element_bytes: int) -> tuple:
        if isinstance(shape, RingShape):
            rows = self.slots * shape.kv_heads * shape.capacity * element_bytes
            sizes = (rows * shape.dim, rows * shape.vdim)
        else:
            sizes = (self.slots * shape.taps * shape.channels * 4, self.slots * shape.heads * shape.vdim * shape.state * 4)
        self.bytes += sum(sizes)
        return tuple(runtime.create_buffer(size) for size in sizes)

    @property
    def free_slots(self) -> int:
        return len(self._free)

    def open(self) -> Sequence:
        if not self._free:
            raise StateError(f"all {self.slots} sequence slots are in use")
        sequence = Sequence(self._free.pop())
        self._live.add(sequence.slot)
        return sequence

    def reserve(self, sequence: Sequence, tokens: int) -> None:
        """Checks that `tokens` more tokens fit."""
        if sequence.slot not in self._live:
            raise StateError("the sequence has been closed")
        if sequence.position + tokens > self.max_context:
            raise StateError(f"the sequence would grow to {sequence.position + tokens} tokens, "
                             f"the pool holds {self.max_context}")

    def close(self, sequence: Sequence) -> None:
        if sequence.slot not in self._live:
            raise StateError("the sequence has been closed")
        self._live.remove(sequence.slot)
        self._free.append(sequence.slot)
