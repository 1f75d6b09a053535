"""Small Zalalix configurations with weights made for the tests, and the plain model's logits for
them.

The weights are not the library's random ones: every kind of tensor gets a spread that makes its
mechanism count (norm weights away from one, biases of the size of the projections, decays that differ
from token to token and from channel to channel, queries and keys whose scores reach the cap), and all
are rounded to bfloat16 first, so that both runtimes and the plain model read the same numbers.  The
configurations differ from each other in every size, and none has two sizes equal that the code could
mix up (key and value sizes, heads and KV heads, the rotated part and the head, windows and pages)."""
from __future__ import annotations

import numpy as np
import torch

from begopel_tiny import distance, load, write_folder  # noqa: F401  (the same helpers serve every design)


def slowed(factor, low, high, original):
    return dict(factor=factor, low=low, high=high, original=original)


def rotation(dims, base=10000.0, scaling=None):
    rot = dict(base=base, dims=dims)
    if scaling is not None:
        rot["scaling"] = scaling
    return rot


def windowed(heads, kv_heads, dim, vdim, scale, size, keep_first, rot, softcap=8.0):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, softcap=softcap, mask=dict(size=size, keep_first=keep_first),
                rot=rot)


def gla(heads, dim, vdim, tau, rank):
    return dict(heads=heads, dim=dim, vdim=vdim, tau=tau, rank=rank)


def parallel(left, right, left_scale=0.7, right_scale=1.3):
    return "parallel", dict(left=left, left_scale=left_scale, right=right, right_scale=right_scale)


def lightning(dim, vdim, decay):
    return "lightning", dict(heads=len(decay), dim=dim, vdim=vdim, decay=list(decay))


def retention(dim, vdim, decay):
    return "retention", dict(heads=len(decay), dim=dim, vdim=vdim, decay=list(decay))


def layer(mixer, ff=None):
    kind, m = mixer
    return dict(type=kind, mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff))


def config(vocab, width, layers, eps=1e-6, scale=3.0):
    return dict(architecture="Zalalix", vocab=vocab, width=width, embedding=dict(scale=scale), norm=dict(eps=eps), layers=layers)


# A: every mixer, with and without a feed-forward; a window that is no multiple of a page, few kept tokens
CONFIG_A = config(211, 72, [
    layer(parallel(windowed(6, 2, 20, 12, 0.25, 37, 5, rotation(8, 5000.0, slowed(4.0, 1.0, 3.0, 64))), gla(3, 10, 14, 4.0, 6)), 40),
    layer(retention(12, 20, [0.9, 0.995]), None),
    layer(lightning(18, 10, [0.5, 0.98, 0.999]), 56),
    layer(parallel(windowed(3, 3, 14, 18, 0.4, 70, 3, rotation(14, 300.0)), gla(2, 24, 8, 1.0, 3), 1.4, -0.6), None),
], eps=1e-5)

# B: sizes of real layers' kind, which the matrix-core attention takes in bfloat16 (keys of 64, 96 and 128, values of
# 64 to 128); more kept tokens than a page holds, and a window shorter than what is kept
CONFIG_B = config(515, 256, [
    layer(lightning(64, 32, [0.7, 0.97, 0.9995, 1.0]), 192),
    layer(parallel(windowed(8, 2, 64, 96, 0.2, 100, 9, rotation(32, 30000.0, slowed(8.0, 1.0, 4.0, 512)), 30.0), gla(3, 44, 40, 12.0, 12)), 320),
    layer(parallel(windowed(4, 4, 96, 64, 0.15, 60, 75, rotation(96, 100000.0), 12.0), gla(2, 64, 128, 2.0, 8), 0.9, 1.0), None),
    layer(retention(32, 64, [0.9375, 0.999, 0.8]), 128),
    layer(parallel(windowed(8, 1, 128, 128, 0.1, 129, 1, rotation(64, 30000.0)), gla(1, 100, 60, 8.0, 20), 1.0, 0.5), 64),
], scale=16.0)

# C: no size is a multiple of 8; one head; windows of one and two positions; nothing kept; a rank of one; decays of nought and one
CONFIG_C = config(77, 50, [
    layer(parallel(windowed(1, 1, 6, 9, 0.5, 1, 2, rotation(2, 50.0)), gla(1, 5, 7, 3.0, 1)), 13),
    layer(lightning(11, 7, [0.0, 0.9, 0.6]), None),
    layer(parallel(windowed(3, 1, 7, 5, 0.4, 2, 0, rotation(6, 10.0, slowed(2.0, 1.0, 2.0, 20)), 2.0), gla(3, 3, 9, 1.0, 5), 1.0, 1.0), 6),
    layer(retention(13, 3, [1.0, 0.25, 0.95]), 9),
], eps=1e-4, scale=1.0)

CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C}


def tensor_shapes(cfg: dict) -> dict:
    """Names and shapes of a configuration's tensors, written out from the design's naming (the
    library's own list is held against this one)."""
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D), "head": (cfg["vocab"], D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        p, q, m = f"l{i}.", f"l{i}.mix.", l["mixer"]
        out.update({p + "norm1": (D,), p + "norm1b": (D,)})

        def state_mixer(q, m):
            qk, vv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({q + "q": (qk, D), q + "k": (qk, D), q + "v": (vv, D), q + "g": (vv, D), q + "o": (D, vv)})
        if l["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            L, R = q + "left.", q + "right."
            out.update({L + "q": (H * d, D), L + "k": (G * d, D), L + "v": (G * dv, D), L + "g": (H, D), L + "o": (D, H * dv), L + "q.b": (H * d,),
                        L + "k.b": (G * d,), L + "v.b": (G * dv,), L + "o.b": (D,), L + "q.norm": (H * d,), L + "k.norm": (G * d,)})
            state_mixer(R, r)
            qk = r["heads"] * r["dim"]
            out.update({R + "a1": (r["rank"], D), R + "a2": (qk, r["rank"]), R + "a2.b": (qk,), R + "norm": (r["vdim"],)})
        else:
            state_mixer(q, m)
            if l["type"] == "lightning":
                out[q + "norm"] = (m["heads"] * m["vdim"],)
        if l["mlp"]:
            ff = l["mlp"]["ff"]
            out.update({p + "norm2": (D,), p + "norm2b": (D,), p + "mlp.gate": (ff, D), p + "mlp.up": (ff, D), p + "mlp.down": (D, ff)})
    return out


def make_weights(cfg: dict, seed: int) -> dict:
    """bfloat16 tensors by name."""
    gen = torch.Generator().manual_seed(seed)
    randn = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if name == "embed":
            t = randn(*shape)
        elif last in ("norm", "norm1", "norm2", "norm1b", "norm2b"):
            t = 1.0 + 0.25 * randn(*shape)
        elif name.endswith("a2.b"):
            t = 1.0 + 1.5 * randn(*shape)                             # decays from strong to hardly any
        elif last == "b":
            t = 0.6 * randn(*shape)                                   # as large as the projections themselves
        elif last == "a2":
            t = 1.5 * randn(*shape) / shape[1] ** 0.5
        elif last == "g":
            t = 1.5 * randn(*shape) / shape[1] ** 0.5
        elif name == "head":
            t = randn(*shape) / shape[1] ** 0.5
        else:
            t = randn(*shape) / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def as_arrays(weights: dict) -> dict:
    return {k: v.to(torch.float64).numpy() for k, v in weights.items()}


def plain_logits(cfg: dict, weights: dict, tokens) -> np.ndarray:
    from plain import zalalix_plain as P
    return P.forward(cfg, as_arrays(weights), list(tokens))


# in 32-bit the engine's sums differ from the plain model's double precision by rounding alone; in
# bfloat16 every product's input is rounded to eight bits
LIMIT = {"float32": 1e-4, "bfloat16": 0.08}
DISTURBANCE = {"float32": 2e-6, "bfloat16": 4e-3}


def row_distances(got, want) -> np.ndarray:
    """Per row what `distance` measures of the worst row."""
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(want)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    spread = np.sqrt(((want - want.mean(-1, keepdims=True)) ** 2).mean())
    return np.sqrt((d ** 2).mean(-1)) / spread


class Truth:
    """The plain model's logits of a sequence, and per row and dtype how far rounding may move them: a
    head's output that is nearly nought before its norm (a query at right angles to the keys) makes a
    large error of a small one, so a row's limit is at least three times what the plain model itself
    shows when the rows that its sublayers read are disturbed by about a rounding each."""

    def __init__(self, cfg: dict, weights: dict, tokens):
        self._args = cfg, as_arrays(weights), list(tokens)
        self.logits = plain_logits(cfg, weights, tokens)
        self._limits = {}

    def __getitem__(self, rows):
        return self.logits[rows]

    def limits(self, dtype: str) -> np.ndarray:
        if dtype not in self._limits:
            from plain import zalalix_plain as P
            rng = np.random.default_rng(0)
            touch = lambda rows: rows * (1.0 + DISTURBANCE[dtype] * rng.standard_normal(rows.shape))
            moved = [row_distances(P.forward(*self._args, touch=touch), self.logits) for _ in range(2)]
            self._limits[dtype] = np.maximum(LIMIT[dtype], 3.0 * np.max(moved, axis=0))
        return self._limits[dtype]


def near(got, truth: Truth, rows, dtype: str) -> bool:
    """Whether the engine's rows lie within their limits of the plain model's; most of many rows lie far
    inside the common limit whatever a few hard ones do."""
    want, limit = np.atleast_2d(truth[rows]), np.atleast_1d(truth.limits(dtype)[rows])
    d = np.atleast_2d(np.asarray(got, np.float64)) - want
    d = d - d.mean(-1, keepdims=True)
    whole = truth.logits - truth.logits.mean(-1, keepdims=True)
    e = np.sqrt((d ** 2).mean(-1)) / np.sqrt((whole ** 2).mean())
    ok = bool((e <= limit).all()) and (len(e) < 16 or float(np.median(e)) <= LIMIT[dtype] / 2)
    if not ok:
        print(f"worst {(e / limit).max():.2f} of its limit, at row {int(np.argmax(e / limit))}: {e[np.argmax(e / limit)]:.5f}; median {np.median(e):.6f}")
    return ok
