"""Requests and the slots that hold their state.

A slot is one row of every state: cache rows of an attention, recurrent states in fp32, the last inputs of a convolution
and the previous token's input; a layer that runs in several passes has a state per pass.  ``RequestTable`` hands slots out, clears what a new request must find
cleared, and keeps what the host knows of a request: its position and which copy of the two-copy inputs is current.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Hashable


@dataclasses.dataclass
class Request:
    slot: int
    position: int = 0    # tokens already in the state
    flip: int = 0        # current copy of the ``shift`` buffers


class RequestTable:
    def __init__(self, globs: Any):
        self.globs = globs
        self.free = list(range(globs.slots))[::-1]
        self.live: dict[Hashable, Request] = {}

    def open(self, key: Hashable) -> Request:
        if key in self.live:
            raise KeyError(f"request {key!r} is live already")
        if not self.free:
            raise RuntimeError(f"all {self.globs.slots} slots are in use")
        request = Request(self.free.pop())
        # Cache rows need no clearing: a row is read only at positions its own request has written.
        for layer in self.globs.layer_state:
            for name in ("state", "shift"):
                if layer.get(name) is not None:
                    layer[name][request.slot].zero_()
        self.live[key] = request
        return request

    def get(self, key: Hashable) -> Request:
        """The live request of this name, opened at its first use."""
        return self.live[key] if key in self.live else self.open(key)

    def close(self, key: Hashable) -> None:
        self.free.append(self.live.pop(key).slot)
