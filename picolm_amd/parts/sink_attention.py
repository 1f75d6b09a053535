"""Causal softmax attention whose every refinement is an option: biases of the projections, a
rotation of part of every head, an RMS norm of queries and keys per head (with a weight, or to unit
root mean square without one), a learned bias by distance, one more term in the softmax's
denominator (a sink, learned per head or a constant), values of a size of their own or the keys
themselves as values, stretches of positions or a window that bound what a query sees, first tokens that
it sees beside its window, a cap on the scores, queries that grow with the position, keys and values of
another layer, and a gate on the heads before the output projection.

    q, k, v, g = W h (+ b);  q, k <- turned by the position;  q <- rms(q) w_q,  k <- rms(k) w_k     per head
    q <- q (1 + coef ln(floor((p + 1) / every) + 1))                   p: the token's position
    s_ij = scale (q_i . k_j) + rel[bucket(i - j)][head]                j <= i, and floor(i / chunk) = floor(j / chunk)
    p_ij = exp(s_ij) / (exp(sink_head) + sum_j' exp(s_ij'))            the sink is a term of the denominator only
    out  = W_o (concat_heads(sum_j p_ij v_j) * sigmoid(g)) (+ b_o)     g: a number an entry, or one a head

With a cap c the scaled score s becomes c tanh(s / c).  With a window of w positions and f kept first
tokens, query i sees key j <= i if i - j < w or j < f.  The norm of queries and keys may cover all
their heads at once instead of each; then it is taken before the rotation.

The bias table has B rows: one per distance below B/2, then rows spaced evenly in the logarithm of
the distance up to `bias_max`, the last row for everything beyond.  It is expanded once, at load,
into one entry per distance up to `bias_max` and per head; the attention kernels index that by
min(distance, last).
"""
from __future__ import annotations

import math

import torch

from .. import kernels
from ..weights import TensorSpec
from .base import KVRequest, Mixer, Runtime
from .calls import AddRowsArgs, SinkAttentionArgs, emit_library_call
from .linear import Linear


def distance_rows(n_rows: int, bias_max: float) -> list[int]:
    """For every distance 0 .. ceil(bias_max) the row of a table of `n_rows` that holds its bias."""
    half = n_rows // 2
    last = int(math.ceil(bias_max))
    if n_rows > 1 and not bias_max > half:
        raise ValueError(f"a bias table of {n_rows} rows needs bias_max above {half}, got {bias_max}")
    rows = []
    for n in range(last + 1):
        if n < half or n_rows == 1:
            rows.append(min(n, n_rows - 1))
        else:
            steps = math.log(n / half) / math.log(bias_max / half) * (n_rows - half)
            rows.append(min(n_rows - 1, half + int(math.floor(steps))))
    return rows


class SinkAttention(Mixer):
    graph_safe = True      # launches depend on device memory only

    def __init__(self, prefix: str, hidden_size: int, n_heads: int, n_kv_heads: int, head_dim: int, v_head_dim: int,
                 scale: float, eps: float, bias_rows: int | None = None, bias_max: float = 0.0, has_bias: bool = False,
                 qk_norm: bool = True, sink: bool = True, gate: bool = True, proj_bias: bool = False, position=None,
                 unit_qk: bool = False, fixed_sink: float | None = None, chunk: int = 0, values_are_keys: bool = False,
                 norm_all: bool = False, softcap: float = 0.0, window: int = 0, keep_first: int = 0, gate_per_head: bool = False,
                 out_bias: bool = False, q_temp: tuple | None = None, reads_keys: bool = False):
        """`has_bias`: scores get the bias by distance, from a table of `bias_rows` rows (None: as many
        as the checkpoint's tensor has) that reaches to `bias_max`.  `proj_bias`: q, k and v have
        biases, the tensors `<name>.b`.  `position`: a `RotaryEmbedding` over the first entries of
        every query and key head (as many as it was made for).  `unit_qk` (without `qk_norm`): queries
        and keys are divided by their root mean square, after the rotation.  `fixed_sink` (without
        `sink`): the denominator's extra term is exp(fixed_sink) for every head, and no tensor holds
        it.  `chunk` > 0: a query sees the keys of its own stretch of `chunk` positions, counted from
        the sequence's first.  `values_are_keys`: there is no value projection; a token's value is its
        key as projected, before rotation and norm.  `norm_all`: the norm of q and the norm of k each
        cover all heads (weights of the projection's size).  `window`, `keep_first`: what a query sees
        (0: every key); the cache keeps all keys and a decode step visits those that are seen.
        `out_bias`: the output projection has one, the tensor `o.b`.  `q_temp` = (coef, every): the
        factor on the queries (after everything else that makes them).  `reads_keys`: the layer has no
        keys and values of its own and reads the cache entry of another layer call, which keeps the
        same kind of them."""
        if n_heads % n_kv_heads:
            raise ValueError(f"{n_heads} heads do not split over {n_kv_heads} KV heads")
        self.prefix, self.D = prefix, hidden_size
        self.H, self.G, self.d, self.dv = n_heads, n_kv_heads, head_dim, v_head_dim
        self.scale, self.eps = float(scale), float(eps)
        self.has_bias = bool(has_bias or bias_rows)
        self.bias_rows, self.bias_max = (None if bias_rows is None else int(bias_rows)), float(bias_max)
        if self.has_bias and not self.bias_max > 0:
            raise ValueError("a bias by distance needs bias_max, the distance its last row starts at")
        self.qk_norm, self.has_sink, self.has_gate = qk_norm, sink, gate
        if values_are_keys and v_head_dim != head_dim:
            raise ValueError(f"values that are the keys have the keys' size {head_dim}, not {v_head_dim}")
        if position is not None and not 0 < position.head_dim <= head_dim:
            raise ValueError(f"a rotation of {position.head_dim} entries of a head of {head_dim}")
        if chunk < 0:
            raise ValueError(f"stretches of {chunk} positions")
        self.proj_bias, self.position, self.unit_qk = bool(proj_bias), position, bool(unit_qk) and not qk_norm
        self.fixed_sink = None if sink or fixed_sink is None else float(fixed_sink)
        self.chunk, self.values_are_keys = int(chunk), bool(values_are_keys)
        if norm_all and not qk_norm:
            raise ValueError("a norm over all heads needs the norm's weights")
        if window < 0 or keep_first < 0 or (keep_first and not window):
            raise ValueError(f"a window of {window} positions beside {keep_first} kept first tokens")
        if softcap < 0 or (softcap and self.has_bias):
            raise ValueError("a cap on the scores and a bias by distance do not go together")
        self.norm_all, self.softcap, self.window, self.keep_first = bool(norm_all), float(softcap), int(window), int(keep_first)
        self.gate_per_head, self.has_out_bias = bool(gate_per_head) and gate, bool(out_bias)
        if q_temp is not None and not q_temp[1] > 0:
            raise ValueError(f"queries that grow every {q_temp[1]} positions")
        self.q_temp, self.reads_keys = None if q_temp is None else (float(q_temp[0]), float(q_temp[1])), bool(reads_keys)
        own = [] if reads_keys else [("k", n_kv_heads * head_dim)] + ([] if values_are_keys else [("v", n_kv_heads * v_head_dim)])
        self.biased = 1 + len(own)         # matrices of the stacked product that may have a bias
        stacked = [("q", n_heads * head_dim)] + own + ([("g", n_heads if gate_per_head else n_heads * v_head_dim)] if gate else [])
        names, sizes = [prefix + n for n, _ in stacked], [size for _, size in stacked]
        self.proj = Linear(names, sizes, hidden_size)
        self.o = Linear([prefix + "o"], [hidden_size], n_heads * v_head_dim)
        self.q_norm = self.k_norm = self.bias = self.sink = self.in_bias = self.o_bias = None
        self.gives_products = False        # True: a part around this one runs proj and o

    def children(self):
        return ([] if self.gives_products else [self.proj, self.o]) + ([self.position] if self.position is not None else [])

    def prepare(self, runtime: Runtime, max_positions: int) -> None:
        if self.position is not None:
            self.position.prepare(runtime, max_positions)

    def tensor_specs(self):
        specs = []
        if self.qk_norm:
            over_q, over_k = (self.H, self.G) if self.norm_all else (1, 1)
            specs.append(TensorSpec(self.prefix + "q.norm", (over_q * self.d,), init="ones"))
            if not self.reads_keys:
                specs.append(TensorSpec(self.prefix + "k.norm", (over_k * self.d,), init="ones"))
        if self.has_bias:       # (-1: any number of rows; random weights need the number)
            specs.append(TensorSpec(self.prefix + "rel", (self.bias_rows if self.bias_rows is not None else -1, self.H)))
        if self.has_sink:
            specs.append(TensorSpec(self.prefix + "sink", (self.H,)))
        if self.proj_bias:
            specs += [TensorSpec(n + ".b", (size,)) for n, size in zip(self.proj.names[:self.biased], self.proj.out_sizes)]
        if self.has_out_bias:
            specs.append(TensorSpec(self.prefix + "o.b", (self.D,)))
        return specs

    def load(self, fetch, runtime: Runtime) -> None:
        f32 = lambda name: fetch.get(self.prefix + name).to(torch.float32).contiguous()
        if self.qk_norm:
            self.q_norm = f32("q.norm")
            self.k_norm = None if self.reads_keys else f32("k.norm")
        if self.has_bias:
            rel = f32("rel")
            rows = distance_rows(rel.shape[0], self.bias_max)
            self.bias = rel[torch.tensor(rows, device=rel.device)].t().contiguous()   # [H, distances]
        if self.has_sink:
            self.sink = f32("sink")
        elif self.fixed_sink is not None:
            self.sink = torch.full((self.H,), self.fixed_sink, dtype=torch.float32, device=runtime.device)
        if self.has_out_bias:
            self.o_bias = f32("o.b")
        if self.proj_bias:          # one entry per column of the stacked product; the gate's columns get none
            parts = [fetch.get(n + ".b").to(torch.float32) for n in self.proj.names[:self.biased]]
            parts.append(torch.zeros(self.proj.out_size - sum(p.numel() for p in parts), dtype=torch.float32, device=parts[0].device))
            self.in_bias = torch.cat(parts).contiguous()

    def cache_requests(self):
        if self.window:
            return KVRequest(self.G, self.d, self.window, self.dv, keeps_all=True, keep_first=self.keep_first), None
        return KVRequest(self.G, self.d, 0, self.dv), None

    def emit(self, b, src, x: int, out_norm=None, out_norm_when: int = 0, accumulate: bool = True) -> None:
        """x (+)= o(gate * attention) for the rows h of `src`, as operations of a launch program."""
        bias = self._emit(b, src, x, kernels.EPI_ACCUMULATE if accumulate else kernels.EPI_STORE,
                          **({"out_norm": out_norm, "out_norm_when": out_norm_when} if accumulate and not self.has_out_bias else {}))
        if bias is not None:
            emit_library_call(b, "add_rows", AddRowsArgs(b._ptr(bias), self.D), x)

    def emit_branch(self, b, src, out: int):
        return self._emit(b, src, out, kernels.EPI_STORE)

    def _emit(self, b, src, x: int, epilogue: int, **norm):
        rows = b.buffer("sink_attn.in", self.proj.out_size, torch.float32)
        self.proj.emit(b, src, rows, kernels.EPI_STORE)
        out = b.buffer("sink_attn.out", self.heads_width, b.dtype)
        self.emit_heads(b, rows, self.proj.out_size, 0, out)
        self.o.emit(b, out, x, epilogue, **norm)
        return self.o_bias

    @property
    def heads_width(self) -> int:
        return self.H * self.dv

    def emit_heads(self, b, rows: int, stride: int, first_col: int, out: int, out_stride: int = 0, out_off: int = 0, mult: float = 1.0) -> None:
        """The work between the two projections: `rows` hold the stacked projection's columns from
        `first_col` on (rows of `stride` floats); the heads' outputs go to the rows `out`, or with
        out_stride > 0, times `mult`, to columns out_off .. of such rows of out_stride entries."""
        H, G, d, dv = self.H, self.G, self.d, self.dv
        width = stride
        q = b.buffer("sink_attn.q", H * d, b.dtype)
        if b.binding is not None and bool(b.binding.writes) == self.reads_keys:
            raise ValueError(f"{self.prefix}: a layer with keys of its own writes its cache entry, one that reads another's does not")
        q_off, k_off = 0, H * d
        v_off = k_off if self.values_are_keys else k_off + G * d
        gate_off = sum(self.proj.out_sizes[:self.biased]) if self.has_gate else -1
        args = SinkAttentionArgs(H, G, d, dv, width, q_off, k_off, v_off, gate_off, self.scale, self.eps,
                                 b._ptr(self.q_norm), b._ptr(self.k_norm), b._ptr(self.bias),
                                 0 if self.bias is None else self.bias.shape[1], b._ptr(self.sink))
        args.chunk, args.unit_qk, args.in_bias = self.chunk, int(self.unit_qk), b._ptr(self.in_bias)
        args.norm_all, args.softcap, args.keep_first, args.gate_per_head = int(self.norm_all), self.softcap, self.keep_first, int(self.gate_per_head)
        args.first_col, args.out_stride, args.out_off, args.out_mult = first_col, out_stride, out_off, mult
        if self.q_temp is not None:
            args.temp_coef, args.temp_every = self.q_temp
        if self.position is not None:
            cos, sin, style = self.position.rotary_tables()
            if cos is None:
                raise ValueError(f"the rotation of {self.prefix} has no tables laid out (prepare)")
            args.cos_table, args.sin_table, args.table_positions = b._ptr(cos), b._ptr(sin), cos.shape[0]
            args.rot_dims, args.rot_half = self.position.head_dim, style
        lib = kernels.lib()
        on_matrix_cores = b.dtype == torch.bfloat16 and lib.picolm_attn_plain_mfma_takes(d, dv)
        emit_library_call(b, "sink_attention", args, out, inp=rows, extra=[q], uses_kv=True, attends=True,
                          tile_rows=lib.picolm_attn_plain_mfma_tile_rows() if on_matrix_cores else kernels.attn_prefill_tile_rows(),
                          partial_floats=H * (dv + 2))
