"""Linear attention whose memory of a sequence is a float32 matrix per head that decays from token to token:

    S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t      (S head_dim x v_dim, zero before the first token)
    x  += out_scale * W_o ((o / rms(o) a head) (* w) * silu(W_g h))

``retention``: alpha is one constant number per head (``decay``), q and k are turned by the nested position part
(rotate-half pairs), k is multiplied by head_dim^(-1/2); the heads' norm has no weight.

``gated_linear_attention``: a decay per head and key channel, alpha = sigmoid(W_a2 (W_a1 h) + b)^(1/tau); q is
multiplied by head_dim^(-1/2); the norm's weight has v_dim numbers that the heads share.

``lightning``: alpha is one constant number per head, q, k and v are the silu of their products; all heads side by side
are RMS-normed together (one root mean square, a weight as long as the row) and multiplied by sigmoid(W_g h).

The input projections are stacked into one matrix, so a step runs one product; its rows leave in float32 and
everything that follows up to the output product's operand is float32: rotation, the decays' second product, their
logarithms and exponentials, the state, the read-out, the norm and the gate.  The state is per-sequence state of the
cache (a row per slot, zeroed when the slot is handed out, moved on by every step), so prompts cut into steps,
batches and decoding all run the same recurrence, to the bit in the 32-bit path.  With bfloat16 activations a step
that brings a sequence more rows than a chunk takes the scan's chunked form on the matrix cores (float32 throughout;
it differs from the walk by rounding); the 32-bit path always walks.

``side_by_side``: two mixers that read the same input and meet as weight * (n(left) + n(right)), n the RMS norm over
the model's width with a weight of its own, or, without norms, as a left + b right (``weight`` a pair of numbers).  Their input matrices are stacked into one product; the pass that joins
the block's branches norms both results.  At most one of the two keeps keys and values; states of both are kept
under "left." and "right.".  Any two mixers that can take their stacked product's rows (``given_input``,
``input_weight``, ``takes_slices``, ``from_rows``) fit.
"""
from __future__ import annotations

from dataclasses import replace

import torch

from .. import ops
from .base import Joined, Mixer, StateSpec, register_part
from .linear import Linear
from .spec import PartSpec, TensorSpec

NAMES = {"q": "q", "k": "k", "v": "v", "gate": "g", "out": "o", "norm": "norm", "decay_down": "a1", "decay_up": "a2",
         "decay_bias": "a2.b"}


def _stack(ws):
    return torch.cat(ws if all(w.dtype == ws[0].dtype for w in ws) else [w.float() for w in ws], dim=0)


def _tensors(prefix, nm, width, heads, head_dim, v_dim):
    qk, vw = heads * head_dim, heads * v_dim
    return {"q": TensorSpec(prefix + nm["q"], (qk, width)), "k": TensorSpec(prefix + nm["k"], (qk, width)),
            "v": TensorSpec(prefix + nm["v"], (vw, width)), "gate": TensorSpec(prefix + nm["gate"], (vw, width)),
            "out": TensorSpec(prefix + nm["out"], (width, vw))}


def retention_spec(prefix: str, width: int, heads: int, head_dim: int, v_dim: int, decay, eps: float, position: PartSpec,
                   out_scale: float = 1.0, names: dict = None, given_input: bool = False) -> PartSpec:
    """``decay``: a number a head."""
    nm = dict(NAMES, **(names or {}))
    return PartSpec("mixer", "retention", {
        "width": width, "heads": heads, "head_dim": head_dim, "v_dim": v_dim, "decay": [float(d) for d in decay],
        "eps": float(eps), "out_scale": float(out_scale), "given_input": bool(given_input)},
        _tensors(prefix, nm, width, heads, head_dim, v_dim), {"position": position})


def lightning_spec(prefix: str, width: int, heads: int, head_dim: int, v_dim: int, decay, eps: float, out_scale: float = 1.0,
                   names: dict = None, given_input: bool = False) -> PartSpec:
    """``decay``: a number a head."""
    nm = dict(NAMES, **(names or {}))
    tensors = _tensors(prefix, nm, width, heads, head_dim, v_dim)
    tensors["norm"] = TensorSpec(prefix + nm["norm"], (heads * v_dim,), init=(1.0, 0.02))
    return PartSpec("mixer", "lightning", {
        "width": width, "heads": heads, "head_dim": head_dim, "v_dim": v_dim, "decay": [float(d) for d in decay],
        "eps": float(eps), "out_scale": float(out_scale), "given_input": bool(given_input)}, tensors)


def gated_linear_attention_spec(prefix: str, width: int, heads: int, head_dim: int, v_dim: int, tau: float, eps: float,
                                rank: int = -1, out_scale: float = 1.0, names: dict = None,
                                given_input: bool = False) -> PartSpec:
    """``rank``: the inner size of the decays' two-step projection; -1 takes what the file's tensors have."""
    nm = dict(NAMES, **(names or {}))
    tensors = _tensors(prefix, nm, width, heads, head_dim, v_dim)
    tensors["norm"] = TensorSpec(prefix + nm["norm"], (v_dim,), init=(1.0, 0.02))
    tensors["decay_down"] = TensorSpec(prefix + nm["decay_down"], (rank, width))
    tensors["decay_up"] = TensorSpec(prefix + nm["decay_up"], (heads * head_dim, rank), init=(0.0, 0.2))
    tensors["decay_bias"] = TensorSpec(prefix + nm["decay_bias"], (heads * head_dim,), init=(2.0, 1.0))
    return PartSpec("mixer", "gated_linear_attention", {
        "width": width, "heads": heads, "head_dim": head_dim, "v_dim": v_dim, "tau": float(tau), "eps": float(eps),
        "out_scale": float(out_scale), "given_input": bool(given_input)}, tensors)


class _DecayMixer(Mixer):
    """What the kinds share: the stacked input product [q | k | v | g | further], the state, the output product."""
    fuses_norm = True
    graph_safe = True     # its launches depend on device buffers only

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        p = spec.params
        self.heads, self.head_dim, self.v_dim = int(p["heads"]), int(p["head_dim"]), int(p["v_dim"])
        self.eps, self.out_scale = float(p["eps"]), float(p.get("out_scale", 1.0))
        limit = ops.decay_scan_max_side()
        if self.head_dim > limit or self.v_dim > limit:
            raise ValueError(f"a state of {self.head_dim} x {self.v_dim} a head is more than the scan kernel's {limit} x {limit}")
        self.qk_width, self.v_width = self.heads * self.head_dim, self.heads * self.v_dim
        stacked = _stack([tensors["q"], tensors["k"], tensors["v"], tensors["gate"]] + self.further_inputs(tensors))
        self.input_weight = stacked if p.get("given_input") else None
        self.inp = None if p.get("given_input") else Linear(stacked, None, rt.fast_kernels)
        self.out = Linear(tensors["out"], None, rt.fast_kernels)
        # the chunked form takes a step's rows in runs of this many (the context lists them)
        self.chunk = ops.decay_chunk_rows(self.head_dim) if rt.act_dtype != torch.float32 and stacked.is_cuda else 0
        self.row_tile = self.chunk or None

    def _chunks(self, ctx):
        return ctx.row_tiles(self.chunk) if self.chunk and ctx.max_new > self.chunk else None

    def further_inputs(self, tensors):
        return []

    def finish_build(self) -> None:
        self.input_weight = None

    def state_spec(self):
        return StateSpec((self.heads, self.head_dim, self.v_dim), torch.float32)

    def _cut(self, rows):
        qk, vw = self.qk_width, self.v_width
        return rows.narrow(-1, 0, qk), rows.narrow(-1, qk, qk), rows.narrow(-1, 2 * qk, vw), rows.narrow(-1, 2 * qk + vw, vw)

    def takes_slices(self, ctx) -> bool:
        """Whether from_rows() adds a product's K slices itself (the walk does)."""
        return self._chunks(ctx) is None

    def _rows(self, h, ctx):
        """The stacked product: in K slices where a kernel cuts K over the grid and the scan adds them, else whole."""
        part = self.inp.partial(h) if self.takes_slices(ctx) else None
        return part if part is not None else self.inp(h, torch.float32)

    def from_rows(self, rows, ctx, binding):
        raise NotImplementedError

    def forward(self, h, x, ctx, binding, then_norm=None):
        y = self.from_rows(self._rows(h, ctx), ctx, binding)
        return self.out.add_into(y, x, then_norm, self.rt.act_dtype, scale=self.out_scale)

    def produce(self, h, ctx, binding):
        """The mixer's result in float32 (whole, or in K slices), for a block that adds it up itself."""
        if self.out_scale != 1.0:
            raise ValueError("a mixer that hands its result over has no multiplier of its own")
        return self.out.raw(self.from_rows(self._rows(h, ctx), ctx, binding))


@register_part("mixer", "retention")
class Retention(_DecayMixer):
    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        decay = spec.params["decay"]
        if len(decay) != self.heads:
            raise ValueError(f"{len(decay)} decays for {self.heads} heads")
        self.decay = torch.tensor(decay, dtype=torch.float32, device=rt.device)
        self.position = parts["position"]
        tables = self.position.rotary_tables()
        if tables is None or tables[1] is not None or self.position.interleaved or getattr(self.position, "magnitude", 1.0) != 1.0:
            raise ValueError("retention takes no rotation, or the rotate-half one by plain frequencies")
        self.inv_freq, _, rot_dims = tables
        self.rot_dims = rot_dims if self.inv_freq is not None else 0
        self.turns = None if self.inv_freq is None else ("angles", tuple(self.inv_freq.tolist()))

    def _angles(self, ctx):
        """The step's cosines and sines: one table for all mixers that turn alike."""
        shared = ctx.shared if ctx.shared is not None else {}
        if self.turns not in shared:
            shared[self.turns] = ops.angle_table(ctx.row_pos, self.inv_freq, ctx.n_rows)
        return shared[self.turns]

    def from_rows(self, rows, ctx, binding):
        """What the output product reads, from the stacked product's float32 rows (a column range of wider rows, or K
        slices of them)."""
        q, k, v, g = self._cut(rows)
        chunks = self._chunks(ctx)
        angles = self._angles(ctx) if chunks is not None and self.turns is not None else None
        return ops.decay_scan(q, k, v, g, binding.state, ctx, self.heads, self.head_dim, self.v_dim, self.eps, self.rt.act_dtype,
                              decay=self.decay, k_scale=self.head_dim ** -0.5, inv_freq=self.inv_freq, rot_dims=self.rot_dims,
                              chunks=chunks, angles=angles)


@register_part("mixer", "lightning")
class Lightning(_DecayMixer):
    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        decay = spec.params["decay"]
        if len(decay) != self.heads:
            raise ValueError(f"{len(decay)} decays for {self.heads} heads")
        self.decay = torch.tensor(decay, dtype=torch.float32, device=rt.device)
        self.norm = tensors["norm"].contiguous()

    def from_rows(self, rows, ctx, binding):
        """What the output product reads, from the stacked product's float32 rows (a column range of wider rows, or K
        slices of them)."""
        q, k, v, g = self._cut(rows)
        o = ops.decay_scan(q, k, v, None, binding.state, ctx, self.heads, self.head_dim, self.v_dim, 0.0, torch.float32,
                           decay=self.decay, chunks=self._chunks(ctx), act_in=True)
        return ops.rownorm_gate(o, self.norm, self.eps, g, self.rt.act_dtype)


@register_part("mixer", "gated_linear_attention")
class GatedLinearAttention(_DecayMixer):
    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        tau = float(spec.params["tau"])
        if tau <= 0:
            raise ValueError("a decay's root must be positive")
        self.rate = 1.0 / tau
        up = tensors["decay_up"]
        self.rank = int(up.shape[1])
        if tensors["decay_down"].shape[0] != self.rank:
            raise ValueError(f"the decays' inner sizes {tensors['decay_down'].shape[0]} and {self.rank} differ")
        self.decay_up = up.float().t().contiguous()                # [rank, heads * head_dim]
        self.decay_bias = tensors["decay_bias"].float().contiguous()
        self.norm = tensors["norm"].contiguous()

    def further_inputs(self, tensors):
        return [tensors["decay_down"]]

    def takes_slices(self, ctx) -> bool:
        return super().takes_slices(ctx) and self.rank <= ops.decay_scan_max_rank()

    def from_rows(self, rows, ctx, binding):
        """What the output product reads, from the stacked product's float32 rows (a column range of wider rows, or K
        slices of them)."""
        q, k, v, g = self._cut(rows)
        first = 2 * (self.qk_width + self.v_width)
        return ops.decay_scan(q, k, v, g, binding.state, ctx, self.heads, self.head_dim, self.v_dim, self.eps, self.rt.act_dtype,
                              decay_from=(rows.narrow(-1, first, self.rank), self.decay_up, self.decay_bias, self.rate), weight=self.norm, q_scale=self.head_dim ** -0.5, chunks=self._chunks(ctx))


def side_by_side_spec(left: PartSpec, right: PartSpec, width: int, eps: float = 0.0, left_norm: str = None, right_norm: str = None,
                      weight=0.5) -> PartSpec:
    """``left``, ``right``: mixers made with ``given_input``; ``left_norm``, ``right_norm``: the names of their norms' weights
    (None: the result is not normed); ``weight``: one number for both, or a pair."""
    for p in (left, right):
        if not p.params.get("given_input"):
            raise ValueError("mixers side by side are handed their stacked product's rows (given_input)")
    weight = tuple(float(w) for w in weight) if isinstance(weight, (tuple, list)) else float(weight)
    norms = {role: TensorSpec(name, (width,), init=(1.0, 0.02)) for role, name in (("left_norm", left_norm), ("right_norm", right_norm))
             if name is not None}
    return PartSpec("mixer", "side_by_side", {"width": width, "eps": float(eps), "weight": weight}, norms,
                    {"left": left, "right": right})


@register_part("mixer", "side_by_side")
class SideBySide(Mixer):
    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        p = spec.params
        self.eps = float(p["eps"])
        self.weights = p["weight"] if isinstance(p["weight"], tuple) else (p["weight"], p["weight"])
        self.left, self.right = parts["left"], parts["right"]
        self.sides = (("left", self.left), ("right", self.right))
        self.norms = (tensors.get("left_norm"), tensors.get("right_norm"))
        if sum(m.cache_spec() is not None for _, m in self.sides) > 1:
            raise ValueError("at most one of two mixers side by side keeps keys and values")
        ws = [m.input_weight for _, m in self.sides]
        self.split = int(ws[0].shape[0])
        self.inp = Linear(_stack(ws), None, rt.fast_kernels)
        for _, m in self.sides:
            m.finish_build()
        self.graph_safe = all(getattr(m, "graph_safe", False) for _, m in self.sides)
        heights = set()
        for _, m in self.sides:
            asked = getattr(m, "row_tile", 0) or ()
            heights.update((asked,) if isinstance(asked, int) else asked)
        self.row_tile = tuple(sorted(heights))

    def cache_spec(self):
        return next((c for c in (m.cache_spec() for _, m in self.sides) if c is not None), None)

    def state_spec(self):
        out = {}
        for name, m in self.sides:
            own = m.state_spec()
            for key, one in (own.items() if isinstance(own, dict) else [("", own)] if own is not None else []):
                out[f"{name}.{key}"] = one
        return out or None

    def _binding(self, name, binding):
        """The binding as one of the two mixers sees it: its own states under their own names."""
        own = {k[len(name) + 1:]: v for k, v in (binding.states or {}).items() if k.startswith(name + ".")}
        return replace(binding, state=own.get(""), states=own)

    def produce(self, h, ctx, binding):
        """Both results, each with its norm, for the pass that joins a block's branches."""
        rows = self.inp.partial(h) if all(m.takes_slices(ctx) for _, m in self.sides) else None
        if rows is None:
            rows = self.inp(h, torch.float32)
        cut = (rows[..., :self.split], rows[..., self.split:])
        out = []
        for (name, m), part, norm, weight in zip(self.sides, cut, self.norms, self.weights):
            y = m.out.raw(m.from_rows(part, ctx, self._binding(name, binding)))
            out.append(Joined(y, weight, norm, self.eps))
        return out

    def forward(self, h, x, ctx, binding):
        ops.join(x, x, [t.term() for t in self.produce(h, ctx, binding)], self.rt.act_dtype, self.eps)
