"""Two mixers as branches of one input.

ParallelMixer: each branch's output is RMS-normed over the model width with a weight of its own, and
the mean of the two joins the residual rows:
    x += 1/2 (rms(left(h)) w_left + rms(right(h)) w_right)
ScaledParallelMixer: the branches are summed with a factor each,
    x += scale_left left(h) + scale_right right(h)
as two products in all: the branches' input projections are stacked into one product over h, and
their output projections lie side by side in one product over [scale_left heads_left | scale_right heads_right].

One branch may ask for keys and values, the other for state; the layer call's cache entry and
state entry serve them."""
from __future__ import annotations

import torch

from .. import kernels
from ..weights import TensorSpec
from .base import Mixer, Runtime
from .calls import AddRowsArgs, NormedSumArgs, emit_library_call
from .linear import JoinedLinear, Linear


def _one_of_each(left: Mixer, right: Mixer) -> tuple:
    lk, ls = left.cache_requests()
    rk, rs = right.cache_requests()
    if (lk is not None and rk is not None) or (ls is not None and rs is not None):
        raise ValueError("two branches that both keep keys and values, or both keep state, need a cache entry each")
    return lk or rk, ls or rs


class ParallelMixer(Mixer):
    graph_safe = True      # launches depend on device memory only

    def __init__(self, left: Mixer, right: Mixer, left_norm: str, right_norm: str, hidden_size: int, eps: float):
        self.left, self.right, self.D, self.eps = left, right, hidden_size, float(eps)
        self.names = (left_norm, right_norm)
        self.w_left = self.w_right = None
        self._requests = _one_of_each(left, right)

    def children(self):
        return [self.left, self.right]

    def tensor_specs(self):
        return [TensorSpec(n, (self.D,), init="ones") for n in self.names]

    def load(self, fetch, runtime: Runtime) -> None:
        self.w_left, self.w_right = (fetch.get(n).to(torch.float32).contiguous() for n in self.names)

    def cache_requests(self):
        return self._requests

    def prepare(self, runtime: Runtime, max_positions: int) -> None:
        self.left.prepare(runtime, max_positions)
        self.right.prepare(runtime, max_positions)

    def emit(self, b, src, x: int, out_norm=None, out_norm_when: int = 0) -> None:
        a = b.buffer("branch.left", self.D, torch.float32)
        c = b.buffer("branch.right", self.D, torch.float32)
        self.left.emit(b, src, a, accumulate=False)
        self.right.emit(b, src, c, accumulate=False)
        emit_library_call(b, "normed_sum", NormedSumArgs(b._ptr(self.w_left), b._ptr(self.w_right), self.D, self.eps, 0.5), x, inp=a,
                          extra=[c])


class ScaledParallelMixer(Mixer):
    """`left` and `right`: mixers whose work between their projections is `emit_heads`, and which hand
    their projections over (`gives_products`)."""
    graph_safe = True      # launches depend on device memory only

    def __init__(self, left: Mixer, right: Mixer, left_scale: float, right_scale: float, hidden_size: int):
        self.left, self.right, self.D = left, right, hidden_size
        self.scales = (float(left_scale), float(right_scale))
        self._requests = _one_of_each(left, right)
        left.gives_products = right.gives_products = True
        self.proj = Linear(left.proj.names + right.proj.names, left.proj.out_sizes + right.proj.out_sizes, hidden_size)
        self.o = JoinedLinear(left.o.names + right.o.names, hidden_size, [left.heads_width, right.heads_width])

    def children(self):
        return [self.proj, self.o, self.left, self.right]

    def cache_requests(self):
        return self._requests

    def prepare(self, runtime: Runtime, max_positions: int) -> None:
        self.left.prepare(runtime, max_positions)
        self.right.prepare(runtime, max_positions)

    def _emit(self, b, src, x: int, epilogue: int, **norm):
        stride, width = self.proj.out_size, self.left.heads_width + self.right.heads_width
        rows = b.buffer("parallel.in", stride, torch.float32)
        self.proj.emit(b, src, rows, kernels.EPI_STORE)
        joined = b.buffer("parallel.heads", width, b.dtype)
        self.left.emit_heads(b, rows, stride, 0, joined, width, 0, self.scales[0])
        self.right.emit_heads(b, rows, stride, sum(self.proj.out_sizes[:len(self.left.proj.names)]), joined, width, self.left.heads_width,
                              self.scales[1])
        self.o.emit(b, joined, x, epilogue, **norm)
        biases = [s * m.o_bias for s, m in zip(self.scales, (self.left, self.right)) if getattr(m, "o_bias", None) is not None]
        return sum(biases[1:], biases[0]).contiguous() if biases else None

    def emit(self, b, src, x: int, out_norm=None, out_norm_when: int = 0, accumulate: bool = True) -> None:
        bias = self._emit(b, src, x, kernels.EPI_ACCUMULATE if accumulate else kernels.EPI_STORE)
        if bias is not None:
            emit_library_call(b, "add_rows", AddRowsArgs(b._ptr(bias), self.D), x)

    def emit_branch(self, b, src, out: int):
        return self._emit(b, src, out, kernels.EPI_STORE)
