"""Small Belorax configurations with weights made for the tests, and the plain model's logits for
them.

The weights are not the library's random ones: every kind of tensor gets a spread that makes its
mechanism count (norm weights away from their neutral values, queries and keys whose scores stand
apart, routers that differ from token to token), and all are rounded to bfloat16 first, so that both
runtimes and the plain model read the same numbers.  The configurations differ from each other in
every size, and none has two sizes equal that the code could mix up (key and value sizes, heads and
KV heads, the rotated part and the head, latents and values, experts and picks).

Every sublayer's output is normed, so a factor on it shows only beside eps: some configurations
have an eps as large as the outputs' squares."""
from __future__ import annotations

import numpy as np
import torch

from begopel_tiny import distance, load, write_folder  # noqa: F401  (the same helpers serve every design)


def yarn(factor, original, fast, slow):
    return dict(factor=factor, original=original, fast=fast, slow=slow)


def rotation(dims, base=10000.0, scaling=None):
    rot = dict(base=base, dims=dims)
    if scaling is not None:
        rot["scaling"] = scaling
    return rot


def retention(dim, vdim, decay, rot):
    return "retention", dict(heads=len(decay), dim=dim, vdim=vdim, decay=list(decay), rot=rot)


def attention(heads, kv_heads, dim, vdim, scale, coef=0.5, every=16, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, q_temp=dict(coef=coef, every=every))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "attention", m


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0, scaling=None):
    return "latent_attention", dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale,
                                    rot=rotation(rot_dim, base, scaling))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff):
    return dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))


def layer(mixer, mlp=None):
    kind, m = mixer
    return dict(type=kind, mixer=m, mlp=mlp)


def config(vocab, width, layers, eps=1e-5, scale=2.0, mult=0.7):
    return dict(architecture="Belorax", vocab=vocab, width=width, embedding=dict(scale=scale), residual_mult=mult, norm=dict(eps=eps), layers=layers)


# A: every mixer with a dense feed-forward, a routed one and none; two layers that read the second one's keys, one of them
# past other layers, with temperatures of their own
CONFIG_A = config(211, 72, [
    layer(retention(14, 20, [0.9, 0.99, 0.5], rotation(8, 300.0)), dense(40)),
    layer(attention(6, 2, 20, 12, 0.4, 0.6, 13), moe(6, 2, 24)),
    layer(attention(6, 2, 20, 12, 0.3, 1.1, 29, kv_from=1), None),
    layer(latent(4, 12, 8, 28, 20, 0.3, 500.0, yarn(4.0, 64, 1.0, 0.25)), moe(5, 3, 16)),
    layer(attention(6, 2, 20, 12, 0.5, 0.0, 7, kv_from=1), dense(56)),
    layer(retention(18, 10, [0.98, 0.999], rotation(18)), None),
], eps=1e-3)

# B: sizes of real layers' kind, which the matrix-core kernels take in bfloat16 (keys of 64, 96 and 128, values of 64 to 128)
CONFIG_B = config(515, 256, [
    layer(attention(8, 2, 64, 96, 0.2, 0.3, 50), moe(8, 3, 64)),
    layer(retention(64, 32, [0.7, 0.97, 0.9995, 1.0], rotation(64, 30000.0)), dense(192)),
    layer(latent(8, 32, 32, 48, 64, 0.12, 100000.0, yarn(8.0, 128, 16.0, 1.0)), moe(4, 1, 128)),
    layer(attention(8, 2, 64, 96, 0.15, 0.8, 31, kv_from=0), None),
    layer(attention(4, 4, 128, 64, 0.1, 0.2, 1), dense(320)),
    layer(latent(6, 64, 64, 128, 64, 0.1, 20000.0, None), dense(64)),
    layer(retention(32, 128, [0.9375, 0.999, 0.8], rotation(16)), moe(16, 16, 32)),
], scale=4.0, mult=1.0)

# C: no size is a multiple of 8; one head; one expert; decays of nought and one; a temperature that grows with every token
CONFIG_C = config(77, 50, [
    layer(latent(1, 5, 2, 7, 9, 0.5, 50.0, yarn(1.5, 20, 3.0, 0.5)), moe(1, 1, 13)),
    layer(attention(1, 1, 7, 5, 0.5, 0.9, 1), dense(21)),
    layer(retention(11, 6, [0.0, 1.0, 0.6], rotation(2, 10.0)), moe(7, 6, 10)),
    layer(attention(1, 1, 7, 5, 0.6, 0.4, 2.5, kv_from=1), None),
    layer(latent(3, 7, 6, 9, 11, 0.4, 10.0, None), None),
], eps=1e-2, scale=1.0, mult=0.9)

CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C}


def tensor_shapes(cfg: dict) -> dict:
    """Names and shapes of a configuration's tensors, written out from the design's naming (the
    library's own list is held against this one)."""
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D), "head": (cfg["vocab"], D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        p, q, m = f"l{i}.", f"l{i}.mix.", l["mixer"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        out.update({p + "norm1": (D,), q + "o": (D, H * dv)})
        if l["type"] == "retention":
            out.update({q + "q": (H * d, D), q + "k": (H * d, D), q + "v": (H * dv, D), q + "g": (H * dv, D)})
        elif l["type"] == "attention":
            out.update({q + "q": (H * d, D), q + "q.norm": (d,)})
            if m.get("kv_from") is None:
                G = m["kv_heads"]
                out.update({q + "k": (G * d, D), q + "v": (G * dv, D), q + "k.norm": (d,)})
        else:
            dr, r = m["rot_dim"], m["kv_rank"]
            out.update({q + "q": (H * (d + dr), D), q + "dkv": (r + dr, D), q + "dkv.norm": (r,), q + "uk": (H * d, r), q + "uv": (H * dv, r)})
        mlp = l["mlp"]
        if not mlp:
            continue
        out[p + "norm2"] = (D,)
        prefixes, ff = [p + "mlp."], mlp.get("ff")
        if mlp["kind"] == "moe":
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            out[p + "mlp.router"] = (E, D)
            prefixes = [f"{p}mlp.e{e}." for e in range(E)]
        for f in prefixes:
            out.update({f + "gate": (ff, D), f + "up": (ff, D), f + "down": (D, ff)})
    return out


def make_weights(cfg: dict, seed: int) -> dict:
    """bfloat16 tensors by name."""
    gen = torch.Generator().manual_seed(seed)
    randn = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        fan = shape[-1] ** 0.5
        if name == "embed":
            t = randn(*shape)
        elif name.endswith(("q.norm", "k.norm", "dkv.norm")):
            t = 1.0 + 0.25 * randn(*shape)
        elif last in ("norm1", "norm2", "norm"):
            t = 0.3 * randn(*shape)                                   # stored around nought
        elif last == "router":
            t = randn(*shape) / fan                                   # (the rows it reads are not normed: they are not small)
        elif name == "head":
            t = randn(*shape) / fan
        else:
            t = randn(*shape) / fan / (cfg["embedding"]["scale"] if last in ("gate", "up", "q", "k", "dkv", "v", "g") else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


def as_arrays(weights: dict) -> dict:
    return {k: v.to(torch.float64).numpy() for k, v in weights.items()}


def plain_logits(cfg: dict, weights: dict, tokens) -> np.ndarray:
    from plain import belorax_plain as P
    return P.forward(cfg, as_arrays(weights), list(tokens))


# in 32-bit the engine's sums differ from the plain model's double precision by rounding alone; in
# bfloat16 every product's input is rounded to eight bits, and a router's logits that lie close
# together may then pick another expert for a token
LIMIT = {"float32": 1e-4, "bfloat16": 0.08}
DISTURBANCE = {"float32": 2e-6, "bfloat16": 4e-3}
CLOSE_CALL = {"float32": 2e-5, "bfloat16": 6e-2}
LOOSE, BEHIND, AFTER = 1.5, 0.35, 8


def row_distances(got, want) -> np.ndarray:
    """Per row what `distance` measures of the worst row."""
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(want)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    spread = np.sqrt(((want - want.mean(-1, keepdims=True)) ** 2).mean())
    return np.sqrt((d ** 2).mean(-1)) / spread


class Truth:
    """The plain model's logits of a sequence, and per row and dtype how far rounding may move them.
    A head's output that is nearly nought before its norm makes a large error of a small one, so a
    row's limit is at least three times what the plain model itself shows when the rows that its
    sublayers read are disturbed by about a rounding each.  A token whose router picked by less than
    CLOSE_CALL is held to LOOSE instead: rounding may give it another expert, and then its row is
    another function's value; later layers' keys and states carry the change on, thinned by the
    other tokens, so the AFTER tokens behind it are held to BEHIND."""

    def __init__(self, cfg: dict, weights: dict, tokens):
        from plain import belorax_plain as P
        self._args = cfg, as_arrays(weights), list(tokens)
        margins = []
        self.logits = P.forward(*self._args, margins=margins)
        self.margins = np.min(margins, axis=0) if margins else np.full(len(tokens), np.inf)
        self._limits = {}

    def __getitem__(self, rows):
        return self.logits[rows]

    def limits(self, dtype: str) -> np.ndarray:
        if dtype not in self._limits:
            from plain import belorax_plain as P
            rng = np.random.default_rng(0)
            touch = lambda rows: rows * (1.0 + DISTURBANCE[dtype] * rng.standard_normal(rows.shape))
            moved = [row_distances(P.forward(*self._args, touch=touch), self.logits) for _ in range(2 if dtype == "float32" else 6)]
            limit = np.maximum(LIMIT[dtype], 3.0 * np.max(moved, axis=0))
            close = self.margins < CLOSE_CALL[dtype]
            behind = np.array([close[max(0, r - AFTER):r].any() for r in range(len(close))])
            limit = np.where(behind, np.maximum(limit, BEHIND), limit)
            self._limits[dtype] = np.where(close, np.maximum(limit, LOOSE), limit)
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
