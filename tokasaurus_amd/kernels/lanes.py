"""A second stream beside the current one, for two pieces of a step's work that do not depend on each other:

    with beside():      # waits for what the current stream has been given so far
        b = ...         # on the second stream
    a = ...             # on the current stream, at the same time
    join()              # the current stream waits for the second

Both streams have the default priority.  Memory needs no care beyond that: what is allocated inside ``beside()`` belongs to the
second stream and is used by the current one behind ``join()``; it is given out again only to later work on the second stream,
which begins by waiting for the current one.  Scratch memory that calls share (``ops.library_workspace``) exists once a lane.
"""

from __future__ import annotations

from contextlib import contextmanager

import torch

_lane = 0
_side: dict[int, torch.cuda.Stream] = {}


def lane() -> int:
    """0 on the current stream, 1 inside ``beside()``."""
    return _lane


def _stream() -> torch.cuda.Stream:
    device = torch.cuda.current_device()
    if device not in _side:
        _side[device] = torch.cuda.Stream(device)
    return _side[device]


@contextmanager
def beside():
    global _lane
    if _lane:
        raise RuntimeError("there is one stream beside the current one")
    side = _stream()
    side.wait_stream(torch.cuda.current_stream())
    _lane = 1
    try:
        with torch.cuda.stream(side):
            yield
    finally:
        _lane = 0


def join() -> None:
    torch.cuda.current_stream().wait_stream(_stream())
