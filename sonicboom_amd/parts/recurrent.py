"""Gated recurrences: mixers whose memory of a sequence is one float32 vector (and, behind a convolution, its last inputs).

``mingru``: the gates read the current token only,

    z_t = sigmoid(W_z h_t + b_z),  u_t = W_x h_t + b_x,
    cand_t = u_t + 1/2 where u_t >= 0, sigmoid(u_t) where u_t < 0,
    S_t = (1 - z_t) S_{t-1} + z_t cand_t   (element by element, S = 0 before the first token),
    x_t += out_scale * W_o (S_t * silu(W_g h_t)).

The three input projections are stacked into one matrix, so a step runs one product; its rows
leave in float32 and the scan kernel takes sigmoid, candidate, update and output gate from there in
float32.  The state is per-sequence state of the cache (one row per slot, zeroed when the slot is
handed out, moved on by every step), so prompts cut into steps, batches and decoding all run the
same recurrence.  In the 32-bit path every step runs the serial kernel, whose sums are those of
token-by-token decoding to the bit; in bfloat16 a step that brings a sequence more rows than a chunk
runs the chunked form.

``gated_lru``: a linear recurrence behind a short causal convolution over time, with gates that are products within equal
blocks of channels,

    u = conv(W_x h + b_x) + b_c,  r = sigmoid(R_a u + b_a),  i = sigmoid(R_i u + b_i)   (block by block),
    a = exp(-8 r softplus(lam)),  S_t = a S_(t-1) + sqrt(1 - a^2) i u,
    x_t += out_scale * W_o (S_t * gelu_tanh(W_y h + b_y)).

W_y and W_x are stacked into one product whose rows leave in float32; everything after it up to the output product's
operand is float32.  The state is S and the convolution's last inputs.  As above the 32-bit path always walks, and
bfloat16 takes the chunked form where a sequence brings more rows than a chunk.
"""
from __future__ import annotations

import torch

from .. import ops
from .base import Mixer, StateSpec, register_part
from .linear import Linear
from .spec import PartSpec, TensorSpec


def mingru_spec(prefix: str, width: int, inner: int, out_scale: float = 1.0) -> PartSpec:
    """Tensors ``<prefix>z``, ``z.b``, ``x``, ``x.b``, ``g``, ``o``."""
    return PartSpec("mixer", "mingru", {"width": width, "inner": inner, "out_scale": float(out_scale)}, {
        "z_weight": TensorSpec(prefix + "z", (inner, width)), "z_bias": TensorSpec(prefix + "z.b", (inner,)),
        "x_weight": TensorSpec(prefix + "x", (inner, width)), "x_bias": TensorSpec(prefix + "x.b", (inner,)),
        "g_weight": TensorSpec(prefix + "g", (inner, width)), "o_weight": TensorSpec(prefix + "o", (width, inner)),
    })


@register_part("mixer", "mingru")
class MinGRU(Mixer):
    fuses_norm = True
    graph_safe = True     # its launches depend on device buffers only

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        p = spec.params
        self.width, self.inner = int(p["width"]), int(p["inner"])
        self.out_scale = float(p.get("out_scale", 1.0))
        ws = [tensors["z_weight"], tensors["x_weight"], tensors["g_weight"]]
        if not all(w.dtype == ws[0].dtype for w in ws):
            ws = [w.float() for w in ws]
        bias = torch.cat([tensors["z_bias"].float(), tensors["x_bias"].float(),
                          torch.zeros(self.inner, dtype=torch.float32, device=ws[0].device)])
        self.zxg = Linear(torch.cat(ws, dim=0), bias, rt.fast_kernels)
        self.out = Linear(tensors["o_weight"], None, rt.fast_kernels)
        # the chunked form takes a step's rows in runs of this many (the context lists them)
        self.chunk = ops.mingru_chunk_rows() if rt.act_dtype != torch.float32 and ws[0].is_cuda else 0
        self.row_tile = self.chunk or None

    def state_spec(self) -> StateSpec:
        return StateSpec((self.inner,), torch.float32)

    def forward(self, h, x, ctx, binding, then_norm=None):
        pre = self.zxg(h, torch.float32)                       # [rows, 3 * inner]: z | x | g before their activations
        chunks = ctx.row_tiles(self.chunk) if self.chunk and ctx.max_new > self.chunk else None
        y = ops.mingru_scan(pre, binding.state, ctx.cu_rows, ctx.slots, ctx.n_seqs, self.rt.act_dtype, chunks)
        return self.out.add_into(y, x, then_norm, self.rt.act_dtype, scale=self.out_scale)


LRU_NAMES = {"y_weight": "y", "y_bias": "y.b", "x_weight": "x", "x_bias": "x.b", "taps": "conv", "taps_bias": "conv.b", "ra": "ra",
             "ra_bias": "ra.b", "ri": "ri", "ri_bias": "ri.b", "lam": "lam", "o_weight": "o"}
LRU_DECAY = 8.0              # what multiplies r softplus(lam)


def gated_lru_spec(prefix: str, width: int, inner: int, blocks: int, taps: int, out_scale: float = 1.0, names: dict = None,
                   given_input: bool = False) -> PartSpec:
    """``inner``: the recurrence's channels, in ``blocks`` equal blocks; ``given_input``: the mixer's stacked input matrix is
    part of a larger one (see ``side_by_side``)."""
    if blocks <= 0 or inner % blocks:
        raise ValueError(f"{blocks} blocks do not divide {inner} channels")
    nm, m = dict(LRU_NAMES, **(names or {})), inner // blocks
    shapes = {"y_weight": (inner, width), "y_bias": (inner,), "x_weight": (inner, width), "x_bias": (inner,), "taps": (inner, taps),
              "taps_bias": (inner,), "ra": (blocks, m, m), "ra_bias": (blocks, m), "ri": (blocks, m, m), "ri_bias": (blocks, m),
              "lam": (inner,), "o_weight": (width, inner)}
    init = {"lam": (-4.5, 1.0), "taps": (0.0, 0.3)}
    return PartSpec("mixer", "gated_lru", {"width": width, "inner": inner, "blocks": blocks, "taps": taps, "out_scale": float(out_scale),
                                           "given_input": bool(given_input)},
                    {role: TensorSpec(prefix + nm[role], shape, init=init.get(role, (0.0, 0.02))) for role, shape in shapes.items()})


@register_part("mixer", "gated_lru")
class GatedLRU(Mixer):
    fuses_norm = True
    graph_safe = True     # its launches depend on device buffers only

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        p = spec.params
        self.width, self.inner, self.taps_n = int(p["width"]), int(p["inner"]), int(p["taps"])
        self.out_scale = float(p.get("out_scale", 1.0))
        block = self.inner // int(p["blocks"])
        most_taps, most_block = ops.gated_lru_limits()
        if not 0 < self.taps_n <= most_taps or block > most_block:
            raise ValueError(f"{self.taps_n} taps and blocks of {block} channels: the recurrence's kernels take {most_taps} and {most_block}")
        ws = [tensors["y_weight"], tensors["x_weight"]]
        stacked = torch.cat(ws if ws[0].dtype == ws[1].dtype else [w.float() for w in ws], dim=0)
        self.input_weight = stacked if p.get("given_input") else None
        self.inp = None if p.get("given_input") else Linear(stacked, None, rt.fast_kernels)
        f32 = lambda role: tensors[role].float().reshape(-1).contiguous()
        self.y_bias, self.x_bias, self.taps_bias = f32("y_bias"), f32("x_bias"), f32("taps_bias")
        self.ra_bias, self.ri_bias = f32("ra_bias"), f32("ri_bias")
        self.taps = tensors["taps"].float().contiguous()
        gates = [tensors["ra"], tensors["ri"]]
        if gates[0].dtype != gates[1].dtype:
            gates = [g.float() for g in gates]
        self.ra, self.ri = (g.contiguous() for g in gates)
        # (a constant of the layer: worked out once, in double)
        self.rate = (LRU_DECAY * torch.nn.functional.softplus(tensors["lam"].double())).float().contiguous()
        self.out = Linear(tensors["o_weight"], None, rt.fast_kernels)
        # the chunked form takes a step's rows in runs of this many (the context lists them)
        chunked = rt.act_dtype != torch.float32 and rt.fast_kernels and stacked.is_cuda and ops.gated_lru_chunked_ok(block, self.ra.dtype)
        self.chunk = ops.gated_lru_chunk_rows() if chunked else 0
        self.row_tile = self.chunk or None

    def finish_build(self) -> None:
        self.input_weight = None

    def state_spec(self):
        return {"state": StateSpec((self.inner,), torch.float32), "inputs": StateSpec((self.taps_n, self.inner), torch.float32)}

    def takes_slices(self, ctx) -> bool:
        """Whether from_rows() adds a product's K slices itself."""
        return True

    def from_rows(self, rows, ctx, binding):
        """What the output product reads, from the stacked product's float32 rows [y | x] (a column range of wider rows, or K
        slices of them)."""
        chunks = ctx.row_tiles(self.chunk) if self.chunk and ctx.max_new > self.chunk else None
        return ops.gated_lru(rows.narrow(-1, self.inner, self.inner), rows.narrow(-1, 0, self.inner), self.x_bias, self.y_bias, self.taps,
                             self.taps_bias, self.ra, self.ri, self.ra_bias, self.ri_bias, self.rate, binding.states["state"],
                             binding.states["inputs"], ctx, self.rt.act_dtype, chunks)

    def _mix(self, h, ctx, binding):
        part = self.inp.partial(h)
        return self.from_rows(part if part is not None else self.inp(h, torch.float32), ctx, binding)

    def forward(self, h, x, ctx, binding, then_norm=None):
        return self.out.add_into(self._mix(h, ctx, binding), x, then_norm, self.rt.act_dtype, scale=self.out_scale)

    def produce(self, h, ctx, binding):
        """The mixer's result in float32 (whole, or in K slices), for a block that adds it up itself."""
        if self.out_scale != 1.0:
            raise ValueError("a mixer that hands its result over has no multiplier of its own")
        return self.out.raw(self._mix(h, ctx, binding))
