"""A second stream beside the current one, for a branch of a layer that meets the other branch at the layer's end.

Small kernels leave most of the chip idle, so two independent chains of them overlap; under graph capture the fork and the
join become edges of the graph.  Everything that runs on the side is forked from and joined to the main stream inside one
layer: memory that a branch frees is handed out again only behind a later fork or join, so no tensor needs to be told about
the other stream."""
from contextlib import contextmanager

import torch

_streams: dict = {}


@contextmanager
def on_the_side(device):
    """Runs its body on the side stream, after what the current stream has been given so far; yields the function that makes
    the current stream wait for it."""
    main = torch.cuda.current_stream(device)
    side = _streams.get(device)
    if side is None:
        side = _streams[device] = torch.cuda.Stream(device)
    side.wait_stream(main)
    with torch.cuda.stream(side):
        yield lambda: main.wait_stream(side)
