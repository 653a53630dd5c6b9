"""Arrangement of norms, mixer and feed-forward in a block.

``prenorm`` (/root/reference/core/src/model/emit.cpp:436-459 without the
optional post-norms): x += mixer(norm(x)); x += ffn(norm(x)).  Mixer and
feed-forward add their result into the float32 residual stream themselves,
which lets their last projection fuse the addition (and a multiplier of the
branch, the ``out_scale`` of their specs).  A block may have no feed-forward:
it is then the first sublayer alone.  With ``input_taps`` the mixer reads h + conv(h) in place of
h = norm(x): a causal convolution over time on every channel of the normed stream (taps
[width, input_taps], the last on the current token, zeros before the sequence's start), whose last
input_taps - 1 inputs are per-sequence state of the block.

``outnorm``: the sublayers read the stream as it is and the norm sits on what they give back:
x += norm(mixer(x)); x += norm(ffn(x)).  The mixer and the feed-forward hand their result over
(``produce``) and one pass sums its slices, norms it, adds it into the stream and leaves the new
stream in the activation type for the sublayer that reads it next.

``parallel``: both sublayers read the same stream, each through a norm of its own, and their results
join it together: x += mixer(norm1(x)) + ffn(norm2(x)).  One pass norms the stream for both (the root
mean square is the same, the weights differ); the mixer and the feed-forward then add into the stream
one after the other.  Without a second norm both sublayers read the first one's result, x += mixer(h) + ffn(h)
with h = norm1(x): they hand their results over (``produce``) and one pass adds the slices of all of
them, norms those that are normed, adds the sum into the stream and leaves what the next block reads.

``streams``: the residual is S streams X_1 .. X_S side by side in a row (hyper-connections).  A sublayer f with its numbers
in [S], out [S] and mix [S, S] (from, to) reads u = sum_s in_s X_s through its norm and leaves
X_t <- sum_s mix[s, t] X_s + out_t f(norm(u)), all t from the old streams.  The sublayers hand their results over
(``produce``); one pass adds the result's slices up, mixes the streams and leaves what the sublayer after it reads, across
the block's end too.
"""
from __future__ import annotations

import torch

from .. import ops
from .base import Branch, Joined, Part, StateSpec, register_part
from .spec import PartSpec, TensorSpec


def prenorm_block_spec(mixer_norm: PartSpec, mixer: PartSpec, ffn_norm: PartSpec = None, ffn: PartSpec = None,
                       input_conv_name: str = None, input_taps: int = 0, width: int = 0) -> PartSpec:
    """``input_conv_name``: the tensor [width, input_taps] of the convolution over time that the
    mixer's input passes (h + conv(h))."""
    parts = {"mixer_norm": mixer_norm, "mixer": mixer}
    if ffn is not None:
        if ffn_norm is None:
            raise ValueError("a block with a feed-forward needs the norm before it")
        parts.update(ffn_norm=ffn_norm, ffn=ffn)
    params, tensors = {}, {}
    if input_conv_name is not None:
        if input_taps < 2 or width <= 0:
            raise ValueError("a convolution on the mixer's input needs at least two taps and the stream's width")
        params = {"input_taps": int(input_taps), "width": int(width)}
        tensors = {"input_conv": TensorSpec(input_conv_name, (width, input_taps), init=(0.0, 0.1))}
    return PartSpec("block", "prenorm", params, tensors, parts)


@register_part("block", "prenorm")
class PreNormBlock(Part):
    category = "block"

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        self.mixer_norm = parts["mixer_norm"]
        self.first_norm = self.mixer_norm      # what the block before may apply in its last pass
        self.mixer = parts["mixer"]
        self.ffn_norm = parts.get("ffn_norm")
        self.ffn = parts.get("ffn")              # None: the block is its mixer's sublayer alone
        self.input_taps = int(spec.params.get("input_taps", 0) or 0)
        self.input_conv = tensors.get("input_conv") if self.input_taps else None
        if self.input_taps and self.input_taps > ops.time_conv_max_taps():
            raise ValueError(f"{self.input_taps} taps are more than the convolution kernel's {ops.time_conv_max_taps()}")

    def state_specs(self):
        """The last taps - 1 inputs of the convolution on the mixer's input, a row of the stream's width each."""
        if not self.input_taps:
            return {}
        return {"input_conv": StateSpec((self.input_taps - 1, int(self.spec.params["width"])), torch.float32)}

    def forward(self, x, ctx, binding, h=None, next_norm=None):
        """Run the block on the residual stream ``x`` in place.  ``h`` is mixer_norm(x) when the
        previous block has already computed it; ``next_norm`` is the norm the next block starts
        with.  Returns next_norm(x) when the feed-forward's last pass produced it, else None.
        Mixers and feed-forwards that can apply a norm in their last pass say so with
        ``fuses_norm``; the others are simply followed by the norm."""
        act = self.rt.act_dtype
        if h is None:
            h = self.mixer_norm.forward(x, act)
        if self.input_conv is not None:
            h = ops.time_conv(h, self.input_conv, None, binding.states["block.input_conv"], ctx, act, residual=True)
        f = None
        after = self.ffn_norm if self.ffn is not None else next_norm     # the norm that follows the mixer
        if getattr(self.mixer, "fuses_norm", False):
            f = self.mixer.forward(h, x, ctx, binding, then_norm=after)
        else:
            self.mixer.forward(h, x, ctx, binding)
        trace = getattr(ctx, "trace", None)
        if trace is not None:
            trace("after_mixer", x)
        if self.ffn is None:
            return f
        if f is None:
            f = self.ffn_norm.forward(x, act)
        out = None
        if getattr(self.ffn, "fuses_norm", False):
            out = self.ffn.forward(f, x, ctx, then_norm=next_norm)
        else:
            self.ffn.forward(f, x, ctx)
        if trace is not None:
            trace("after_ffn", x)
        return out


def outnorm_block_spec(mixer_norm: PartSpec, mixer: PartSpec, ffn_norm: PartSpec = None, ffn: PartSpec = None) -> PartSpec:
    parts = {"mixer_norm": mixer_norm, "mixer": mixer}
    if ffn is not None:
        if ffn_norm is None:
            raise ValueError("a block with a feed-forward needs the norm after it")
        parts.update(ffn_norm=ffn_norm, ffn=ffn)
    return PartSpec("block", "outnorm", {}, {}, parts)


class StreamAsItIs:
    """What a block that reads the stream itself names as its ``first_norm``: no norm, the stream
    in the activation type.  A block before it that cannot produce that in its last pass is simply
    followed by the conversion."""
    fusable = False
    join_kind = "copy"
    weight = None
    eps = 0.0

    def forward(self, x, out_dtype, rows=None):
        if rows is not None:
            raise ValueError("the stream as it is has no picked rows")
        return ops.cast(x, out_dtype)


@register_part("block", "outnorm")
class OutNormBlock(Part):
    category = "block"

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        self.mixer_norm = parts["mixer_norm"]
        self.first_norm = StreamAsItIs()
        self.mixer = parts["mixer"]
        self.ffn_norm = parts.get("ffn_norm")
        self.ffn = parts.get("ffn")
        for part, what in ((self.mixer, "mixer"), (self.ffn, "feed-forward")):
            if part is not None and not hasattr(part, "produce"):
                raise ValueError(f"a block that norms outputs needs a {what} that hands its result over (produce)")
        for n in (self.mixer_norm, self.ffn_norm):
            if n is not None and (getattr(n, "groups", 1) != 1 or not hasattr(n, "eps")):
                raise ValueError("a block that norms outputs takes RMS norms over whole rows")

    def _join(self, x, y, norm, copy_dtype):
        """x += norm(y); the new stream in ``copy_dtype`` (x itself when that is float32)."""
        if isinstance(y, Joined):
            if y.scale != 1.0 or y.norm_weight is not None:
                raise ValueError("a block that norms outputs takes results without a scale or a norm of their own")
            y = Branch(y.part, extra=None if y.bias is None else y.bias.float().expand(x.shape).contiguous())
        b = y if isinstance(y, Branch) else Branch(y)
        return ops.norm_add(x, b.part, norm.weight, norm.eps, getattr(norm, "offset", 0.0), copy_dtype,
                            part_weights=b.part_weights, extra=b.extra, extra_weights=b.extra_weights, by_row=b.by_row)

    def forward(self, x, ctx, binding, h=None, next_norm=None):
        """Run the block on the residual stream ``x`` in place.  ``h``: the stream in the activation
        type when the block before has left it.  Returns the stream in the activation type when the
        next block reads it as it is, else None."""
        act = self.rt.act_dtype
        if h is None:
            left = (getattr(ctx, "shared", None) or {}).pop("stream", None)      # the embedding's own copy of what it made
            h = left[1] if left is not None and left[0] is x and left[1].dtype == act else ops.cast(x, act)
        last = self.ffn is None
        want = act if not last or isinstance(next_norm, StreamAsItIs) else None
        h = self._join(x, self.mixer.produce(h, ctx, binding), self.mixer_norm, want)
        trace = getattr(ctx, "trace", None)
        if trace is not None:
            trace("after_mixer", x)
        if last:
            return h
        want = act if isinstance(next_norm, StreamAsItIs) else None
        h = self._join(x, self.ffn.produce(h, ctx), self.ffn_norm, want)
        if trace is not None:
            trace("after_ffn", x)
        return h


def parallel_block_spec(mixer_norm: PartSpec, mixer: PartSpec, ffn_norm: PartSpec = None, ffn: PartSpec = None) -> PartSpec:
    """``ffn_norm`` None: the feed-forward reads the mixer's norm."""
    parts = {"mixer_norm": mixer_norm, "mixer": mixer}
    if ffn is not None:
        parts["ffn"] = ffn
        if ffn_norm is not None:
            parts["ffn_norm"] = ffn_norm
    return PartSpec("block", "parallel", {}, {}, parts)


def _terms(y):
    """A sublayer's result as terms of the joining pass."""
    if isinstance(y, Joined):
        return [y]
    if isinstance(y, (list, tuple)):
        return [t for one in y for t in _terms(one)]
    return [Joined(y)]


def _one_bias(terms):
    biases = [t.bias for t in terms if t.bias is not None]
    if len(biases) > 1:
        raise ValueError("one of the branches that join in a pass may bring a bias")
    return biases[0] if biases else None


def join_branches(x, results, act_dtype, next_norm=None):
    """x += the sublayers' ``results`` in one pass over the row; next_norm(x) in ``act_dtype`` when that pass can make
    it, else None."""
    terms = []
    for y in results:
        if isinstance(y, Branch):       # slices with a multiplier a row each: a pass of their own, after which they are in x
            ops.norm_add(x, y.part, None, 0.0, 0.0, None, part_weights=y.part_weights, extra=y.extra,
                         extra_weights=y.extra_weights, by_row=y.by_row, norm=False)
        else:
            terms += _terms(y)
    kind = getattr(next_norm, "join_kind", None)
    epses = {t.eps for t in terms if t.norm_weight is not None}
    if len(epses) > 1:
        raise ValueError("the branches of a block are normed with one eps")
    # (the pass takes a few branches; what is more goes first)
    while len(terms) > ops.JOIN_MAX_TERMS:
        first = terms[:ops.JOIN_MAX_TERMS]
        ops.join(x, x, [t.term() for t in first], act_dtype, max(epses, default=0.0), vec=_one_bias(first))
        terms = terms[ops.JOIN_MAX_TERMS:]
    return ops.join(x, x, [t.term() for t in terms], act_dtype, max(epses, default=0.0), vec=_one_bias(terms), then=kind,
                    then_weight=next_norm.weight if kind else None, then_eps=next_norm.eps if kind else 0.0,
                    out_dtype=act_dtype)


@register_part("block", "parallel")
class ParallelBlock(Part):
    category = "block"

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        self.mixer_norm = parts["mixer_norm"]
        self.mixer = parts["mixer"]
        self.ffn_norm = parts.get("ffn_norm")
        self.ffn = parts.get("ffn")              # None: the block is its mixer's branch alone
        # both branches read one norm's result: where both hand their results over, one pass joins them
        self.one_norm = self.ffn is not None and self.ffn_norm is None
        self.joins = all(hasattr(p, "produce") for p in (self.mixer, self.ffn) if p is not None) \
            and (self.one_norm or not hasattr(self.mixer, "fuses_norm"))
        # with two branches the block norms for both in one pass of its own; alone, the mixer's norm is what
        # the block before may apply in its last pass
        self.first_norm = self.mixer_norm if self.ffn is None or self.one_norm else None
        a, b = self.mixer_norm, self.ffn_norm
        # one pass for both norms when they are RMS norms over whole rows with the same eps and plain weights
        self.one_pass = b is not None and all(
            getattr(n, "fusable", False) and getattr(n, "groups", 1) == 1 and hasattr(n, "eps") for n in (a, b)) \
            and a.eps == b.eps and (a.weight is None) == (b.weight is None) \
            and (a.weight is None or a.weight.dtype == b.weight.dtype)

    def forward(self, x, ctx, binding, h=None, next_norm=None):
        """Run the block on the residual stream ``x`` in place.  ``h`` is mixer_norm(x) when the block
        before has already computed it.  Returns next_norm(x) when the last pass produced it, else None.
        Both branches are normed before either result joins the stream."""
        act = self.rt.act_dtype
        f = None
        trace = getattr(ctx, "trace", None)
        if self.one_norm or (self.ffn is None and self.joins):
            if h is None:
                h = self.mixer_norm.forward(x, act)
            out = None
            if self.joins:
                results = [self.mixer.produce(h, ctx, binding)]
                if self.ffn is not None:
                    results.append(self.ffn.produce(h, ctx))
                out = join_branches(x, results, act, next_norm)
            else:
                self.mixer.forward(h, x, ctx, binding)
                self.ffn.forward(h, x, ctx)
            if trace is not None:
                trace("after_mixer" if self.ffn is None else "after_ffn", x)
            return out
        if self.ffn is not None:
            if h is None and self.one_pass:
                h, f = ops.rmsnorm_pair(x, self.mixer_norm.weight, self.ffn_norm.weight, self.mixer_norm.eps, act)
            else:
                f = self.ffn_norm.forward(x, act)
        if h is None:
            h = self.mixer_norm.forward(x, act)
        last = self.ffn is None
        if getattr(self.mixer, "fuses_norm", False):
            out = self.mixer.forward(h, x, ctx, binding, then_norm=next_norm if last else None)
        else:
            out = self.mixer.forward(h, x, ctx, binding)
        if trace is not None:
            trace("after_mixer", x)
        if last:
            return out
        out = None
        if getattr(self.ffn, "fuses_norm", False):
            out = self.ffn.forward(f, x, ctx, then_norm=next_norm)
        else:
            self.ffn.forward(f, x, ctx)
        if trace is not None:
            trace("after_ffn", x)
        return out


def streams_block_spec(streams: int, mixer_norm: PartSpec, mixer: PartSpec, mixer_names: dict, ffn_norm: PartSpec = None,
                       ffn: PartSpec = None, ffn_names: dict = None) -> PartSpec:
    """``mixer_names``, ``ffn_names``: the file's names of a sublayer's "in" [streams], "out" [streams] and "mix"
    [streams, streams]."""
    S = int(streams)
    parts, tensors = {"mixer_norm": mixer_norm, "mixer": mixer}, {}
    if ffn is not None:
        if ffn_norm is None or ffn_names is None:
            raise ValueError("a block with a feed-forward needs the norm before it and its numbers")
        parts.update(ffn_norm=ffn_norm, ffn=ffn)
    for which, names in (("mixer", mixer_names), ("ffn", ffn_names if ffn is not None else None)):
        if names is not None:
            tensors[which + "_in"] = TensorSpec(names["in"], (S,), init=(1.0 / S, 0.1))
            tensors[which + "_out"] = TensorSpec(names["out"], (S,), init=(1.0, 0.1))
            tensors[which + "_mix"] = TensorSpec(names["mix"], (S, S), init=(1.0 / S, 0.1))
    return PartSpec("block", "streams", {"streams": S}, tensors, parts)


class StreamsRead:
    """What a sublayer of a ``streams`` block reads: norm(sum_s read[s] X_s)."""
    fusable = False
    join_kind = None

    def __init__(self, read, norm):
        self.read, self.norm = read, norm
        if getattr(norm, "groups", 1) != 1 or not hasattr(norm, "eps") or not getattr(norm, "fusable", False):
            raise ValueError("a block of several streams takes RMS norms over whole rows with plain weights")


@register_part("block", "streams")
class StreamsBlock(Part):
    category = "block"

    def __init__(self, spec, tensors, parts, rt):
        super().__init__(spec, tensors, parts, rt)
        self.streams = int(spec.params["streams"])
        if not 0 < self.streams <= ops.streams_max():
            raise ValueError(f"{self.streams} streams: the kernels take 1 to {ops.streams_max()}")
        self.mixer, self.ffn = parts["mixer"], parts.get("ffn")
        for part, what in ((self.mixer, "mixer"), (self.ffn, "feed-forward")):
            if part is not None and not hasattr(part, "produce"):
                raise ValueError(f"a block of several streams needs a {what} that hands its result over (produce)")
        self.numbers = {role: t.float().contiguous() for role, t in tensors.items()}
        self.first_norm = StreamsRead(self.numbers["mixer_in"], parts["mixer_norm"])
        self.ffn_read = StreamsRead(self.numbers["ffn_in"], parts["ffn_norm"]) if self.ffn is not None else None

    def _join(self, which, x, y, then):
        terms, biases = [], []
        for one in (y if isinstance(y, (list, tuple)) else [y]):
            if isinstance(one, Branch):
                terms.append((one.part, 1.0, one.by_row, one.part_weights))
                if one.extra is not None:
                    terms.append((one.extra, 1.0, False, one.extra_weights))
                continue
            one = one if isinstance(one, Joined) else Joined(one)
            if one.norm_weight is not None:
                raise ValueError("a block of several streams does not norm its branches")
            terms.append((one.part, one.scale, False, None))
            if one.bias is not None:
                biases.append(one.bias)
        if len(biases) > 1:
            raise ValueError("one of a sublayer's branches may bring a bias")
        read = isinstance(then, StreamsRead)
        return ops.streams_join(x, self.streams, terms, self.numbers[which + "_mix"], self.numbers[which + "_out"],
                                vec=biases[0] if biases else None, read=then.read if read else None,
                                weight=then.norm.weight if read else None, eps=then.norm.eps if read else 0.0,
                                act_dtype=self.rt.act_dtype)

    def forward(self, x, ctx, binding, h=None, next_norm=None):
        """Run the block on the streams ``x`` [rows, streams * width] in place.  ``h``: what the mixer reads when the block
        before has left it.  Returns what the next block's mixer reads when that is a block of several streams too."""
        trace = getattr(ctx, "trace", None)
        if h is None:
            first = self.first_norm
            h = ops.streams_read(x, self.streams, first.read, first.norm.weight, first.norm.eps, self.rt.act_dtype)
        h = self._join("mixer", x, self.mixer.produce(h, ctx, binding), self.ffn_read if self.ffn is not None else next_norm)
        if trace is not None:
            trace("after_mixer", x)
        if self.ffn is None:
            return h
        h = self._join("ffn", x, self.ffn.produce(h, ctx), next_norm)
        if trace is not None:
            trace("after_ffn", x)
        return h
