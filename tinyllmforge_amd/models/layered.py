"""What designs with a list of unlike layers share: rotation tables, the forward loop, checkpoint names, packing.

A layer is a module with what turns the stream into its input (the attribute that ``front`` names: the norm in front of it, or a
token shift), ``forward(positions, h, x, following)`` that updates the fp32 stream ``x`` in place and returns it as ``following``
makes it the next input, and ``routes()``: checkpoint names below ``l<i>.`` ->
(parameter below the layer, part of it or None).  A layer that runs more than once takes ``run=`` (0, 1, ...) and keeps a cache
and a state of its own per run."""
import re
from functools import partial

import torch
from torch import nn

from ..layers.linear import GatedUpLinear, JoinedLinear, StackedLinear
from ..layers.rotary_embedding import rotation_table


def prefixed(prefix: str, routes: dict) -> dict:
    return {prefix + name: (prefix + target, part) for name, (target, part) in routes.items()}


class LayeredForCausalLM(nn.Module):
    front = "norm1"
    fixed_tensors = {"embed": ("embed", None), "final.norm": ("norm.weight", None)}

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.embed = nn.Parameter(torch.empty(config.vocab, config.width))
        self.loaded_tensors: set[str] = set()
        self._rope_tables = {}

    def rope_table(self, rot: dict | None):
        """Layers with the same rotation share a table."""
        if not rot or not rot["dims"]:
            return None
        scaling = rot.get("scaling") or {}
        key = (rot["dims"], rot["base"], *sorted(scaling.items()))
        if key not in self._rope_tables:
            table = rotation_table(rot["dims"], self.config.max_position_embeddings, rot["base"], **scaling)
            self._rope_tables[key] = table.to(self.embed.device)
        return self._rope_tables[key]

    def runs(self):
        """The layers in the order they run, ``(what makes its input, call)``."""
        order, seen = self.config.layer_runs(), {}
        for i in order:
            run = seen[i] = seen.get(i, -1) + 1
            layer = self.layers[i]
            yield getattr(layer, self.front), partial(layer, run=run) if order.count(i) > 1 else layer

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        runs = list(self.runs())
        fronts = [front for front, _ in runs] + [self.norm]
        x, h = fronts[0].after_embedding(input_ids, self.embed.data, positions)
        for (_, layer), following in zip(runs, fronts[1:]):
            h = layer(positions, h, x, following)
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        return self.head(hidden_states)

    def compute_greedy_ids(self, hidden_states: torch.Tensor) -> torch.Tensor:
        return self.head.forward_greedy(hidden_states)

    # -- checkpoint names
    def route_tensor(self, name: str):
        """Checkpoint tensor -> (parameter, part of it or None)."""
        if name in self.fixed_tensors:
            return self.fixed_tensors[name]
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        routes = self.layers[int(m[1])].routes() if m and int(m[1]) < len(self.layers) else {}
        if not m or m[2] not in routes:
            raise KeyError(f"unknown tensor {name!r}")
        target, part = routes[m[2]]
        return f"layers.{m[1]}.{target}", part

    def expected_tensors(self) -> set[str]:
        return set(self.fixed_tensors) | {f"l{i}.{n}" for i, layer in enumerate(self.layers) for n in layer.routes()}

    # -- what the engine does with the weights after loading
    def _linears(self):
        for layer in self.layers:
            yield from (m for m in layer.modules() if isinstance(m, (StackedLinear, JoinedLinear, GatedUpLinear)))

    def quantize_linears_(self):
        """Weight-only int8 for the projections of every layer (embedding, head and experts stay as they are)."""
        for lin in self._linears():
            lin.zero_pads_()
            lin.quantize_()
        return self

    def pack_linears_(self):
        """Once after loading, on the GPU: pads back to zero, then the row and tile orders the fused kernels read."""
        for lin in [*self._linears(), self.head]:
            if not getattr(lin, "interleaved", False):
                lin.zero_pads_()
            if lin.is_quantized:
                lin.pack_()
            elif isinstance(lin, GatedUpLinear) and lin.weight.dtype == torch.bfloat16:
                lin.interleave_()
        return self
