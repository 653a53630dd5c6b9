"""What stands between two blocks of the run order where a model repeats a run of blocks.

``mix_embedding``: x <- W [x; x0] + step[turn], x0 the embedding's output, W [width, 2 width] with x's columns first,
``step`` a vector a pass.  W x0's share of the product does not change from pass to pass: it is made once a step, so a
pass runs the product of x's columns alone, and one pass over the row adds its slices, that share and the vector and
norms the result for the block that follows.
"""
from __future__ import annotations

import torch

from .. import ops
from .base import Part, register_part
from .block import StreamAsItIs
from .linear import Linear
from .spec import PartSpec, TensorSpec


def mix_embedding_spec(mix_name: str, step_name: str, width: int, turns: int) -> PartSpec:
    return PartSpec("junction", "mix_embedding", {"width": width, "turns": int(turns)}, {
        "mix": TensorSpec(mix_name, (width, 2 * width)),
        "step": TensorSpec(step_name, (turns, width), init=(0.0, 0.1))})


@register_part("junction", "mix_embedding")
class MixEmbedding(Part):
    category = "junction"
    graph_safe = True     # its launches depend on device buffers only

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        width = int(spec.params["width"])
        mix = tensors["mix"]
        self.from_x = Linear(mix[:, :width].contiguous(), None, rt.fast_kernels)
        self.from_x0 = Linear(mix[:, width:].contiguous(), None, rt.fast_kernels)
        self.steps = tensors["step"].contiguous()
        self.first_norm = StreamAsItIs()       # the block before may hand over x in the activation type

    def begin(self, x0, ctx):
        """Once a step, before any block has run.  Returns x0 in the activation type."""
        act = self.rt.act_dtype
        left = ctx.shared.get("stream")        # the embedding's own copy of what it made
        h = left[1] if left is not None and left[0] is x0 and left[1].dtype == act else ops.cast(x0, act)
        ctx.shared[self] = self.from_x0(h, torch.float32)
        return h

    def forward(self, x, ctx, turn, next_norm=None, h=None):
        """x is overwritten.  ``h``: x in the activation type when what ran before has left it.  Returns next_norm(x)
        when the last pass could make it, else None."""
        act = self.rt.act_dtype
        ctx.shared.pop("stream", None)         # x changes
        if h is None:
            h = ops.cast(x, act)
        kind = getattr(next_norm, "join_kind", None)
        return ops.join(x, ctx.shared[self], [(self.from_x.raw(h), 1.0, False, None)], act, vec=self.steps[turn], then=kind,
                        then_weight=next_norm.weight if kind else None, then_eps=next_norm.eps if kind else 0.0, out_dtype=act)
