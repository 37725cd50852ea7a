"""Parts of blocks whose residual is several 32-bit streams that are mixed at every sublayer.

The streams X_1 .. X_S travel as a `Stream32` whose `full` is [rows, S, width], or [rows, width] as long as all of them
are equal (the embedding). A sublayer reads u = sum_s read[s] X_s through an RMS norm; its result y joins them all at
once, X_t <- sum_s mix[s, t] X_s + out[t] y. One kernel does a sublayer's end and the next one's beginning: the mix, the
weighted sum, the norm that reads it and, before a mixer, the mix with the row before.
"""
from __future__ import annotations

import torch

from .base import ARRANGEMENTS, CONNECTIONS, NORMS, ROW_SHIFTS, Arrangement, to_gain
from .spec import StateNeed
from .stream32 import Stream32


@NORMS.register("streams_rmsnorm")
class StreamsRmsNorm:
    """y = u / sqrt(mean(u^2) + eps) * gain with u = sum_s read[s] X_s (weighted: false: the plain sum), in 32-bit; rows in
    the compute type. params: width, streams, eps, weighted. tensors: gain (width,), with weighted read (streams,)."""
    graph_safe = True

    @classmethod
    def tensor_shapes(cls, params):
        shapes = {"gain": (params["width"],)}
        if params.get("weighted", True):
            shapes["read"] = (params["streams"],)
        return shapes

    def __init__(self, spec, tensors, ops):
        self.ops = ops
        self.streams, self.eps = int(spec.params["streams"]), float(spec.params["eps"])
        self.gain = to_gain(ops, tensors.of(spec, "gain"))
        self.read = to_gain(ops, tensors.of(spec, "read")) if spec.params.get("weighted", True) else \
            torch.ones(self.streams, dtype=torch.float32, device=ops.device)

    def reading(self):
        """(weights, gain, eps) for a kernel that applies this norm to the streams it has just mixed."""
        return self.read, self.gain, self.eps

    def __call__(self, x):
        if x.normed_by is self:
            return x.rows               # the block before has applied this norm in its last kernel
        return self.ops.mix_streams(x.full, self.streams, read=self.reading())[1]


@CONNECTIONS.register("stream_mix")
class StreamMix:
    """How a sublayer's result y joins the streams: X_t <- sum_s mix[s, t] X_s + out[t] y. params: streams. tensors: mix
    (streams, streams) indexed [from, to], out (streams,)."""
    graph_safe = True

    @classmethod
    def tensor_shapes(cls, params):
        return {"mix": (params["streams"], params["streams"]), "out": (params["streams"],)}

    def __init__(self, spec, tensors, ops):
        self.mix, self.out = to_gain(ops, tensors.of(spec, "mix")), to_gain(ops, tensors.of(spec, "out"))


@ROW_SHIFTS.register("previous_row")
class PreviousRow:
    """h_t <- h_t + (h_(t-1) - h_t) * amount, channel by channel, h_(t-1) being the row before as it was before the shift
    (zeros before a request's first row; kept in 32-bit between steps). params: width. tensors: amount (width,)."""
    graph_safe = True

    @classmethod
    def tensor_shapes(cls, params):
        return {"amount": (params["width"],)}

    @classmethod
    def cache_need(cls, params):
        return StateNeed((params["width"],), "float32")

    def __init__(self, spec, tensors, ops):
        self.amount = to_gain(ops, tensors.of(spec, "amount"))


class Entry:
    """A block's beginning as the block before may run it: a norm of the streams, and the shift behind it."""
    __slots__ = ("norm", "shift", "shift_name")

    def __init__(self, norm, shift, shift_name):
        self.norm, self.shift, self.shift_name = norm, shift, shift_name

    def shifting(self, ctx):
        """(amount, the requests' kept rows, the step's batch) with ctx the entering call's context; None: no shift."""
        return (self.shift.amount, ctx.of(self.shift_name).state, ctx.batch) if self.shift is not None else None


@ARRANGEMENTS.register("hyper_stream32")
class HyperStream32(Arrangement):
    """y = mixer(shift(norm_a(X))), X <- join_a(X, y);  y = feed_forward(norm_f(X)), X <- join_f(X, y), on S streams.

    The shift and the feed-forward (with its norm and connection) are optional. params: streams. parts: mixer_norm and
    feed_forward_norm (kind "streams_rmsnorm"), mixer, feed_forward, mixer_connection, feed_forward_connection, mixer_shift.
    """
    part_names = None

    def __init__(self, layer_spec, tensors, ops):
        super().__init__(layer_spec, tensors, ops)
        need = {"mixer_norm", "mixer", "mixer_connection"}
        second = {"feed_forward_norm", "feed_forward", "feed_forward_connection"}
        have = set(self.parts)
        if not need <= have or have - need - second - {"mixer_shift"} or (have & second and not second <= have):
            raise ValueError(f"a hyper_stream32 block is made of {sorted(need)}, optionally ['mixer_shift'] and all of "
                             f"{sorted(second)}; its spec brings {sorted(have)}")
        self.streams = int(layer_spec.params["streams"])
        self.mixer, self.join_a = self.parts["mixer"], self.parts["mixer_connection"]
        self.ffn, self.norm_f = self.parts.get("feed_forward"), self.parts.get("feed_forward_norm")
        self.join_f = self.parts.get("feed_forward_connection")
        self.first_norm = Entry(self.parts["mixer_norm"], self.parts.get("mixer_shift"), "mixer_shift")

    def _join(self, full, y, bias, join, read=None, shift=None):
        return self.ops.mix_streams(full, self.streams, write=(y, bias, join.mix, join.out), read=read, shift=shift)

    @staticmethod
    def _result(part, *args):
        """(a sublayer's result in 32-bit, the output bias it leaves to the sum or None)"""
        return part.forward_parts(*args) if hasattr(part, "forward_parts") else (part.forward32(*args), None)

    def forward(self, x, ctx):
        full, enter = x.full, self.first_norm
        if x.normed_by is enter:
            h = x.rows
        else:
            h = self.ops.mix_streams(full, self.streams, read=enter.norm.reading(), shift=enter.shifting(ctx))[1]
        y, bias = self._result(self.mixer, h, ctx.of("mixer"))
        join = self.join_a
        if self.ffn is not None:
            full, h = self._join(full, y, bias, self.join_a, read=self.norm_f.reading())
            y, bias = self._result(self.ffn, h)
            join = self.join_f
        # the block's last mix also begins what reads the streams next, where that reads streams
        after = ctx.next_norm
        if isinstance(after, Entry):
            full, h = self._join(full, y, bias, join, read=after.norm.reading(), shift=after.shifting(ctx.next_call))
        elif isinstance(after, StreamsRmsNorm):
            full, h = self._join(full, y, bias, join, read=after.reading())
        else:
            (full, _), h, after = self._join(full, y, bias, join), None, None
        return Stream32(full, h, normed_by=after)
