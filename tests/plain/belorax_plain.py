"""The Belorax decoder as a plain function of a whole sequence, in double precision: one function per
mechanism, no cache, no batching, no kernels.  What the engine computes is held against this.

Notation: h [T, D] rows of one sequence in order; W a dict of arrays by tensor name; weights are
stored [out, in] and applied as W x; positions count from 0.

    x       = scale_e embed[token]
    layer   : x = x + m n1(mixer(x));  x = x + m n2(ff(x))            ff may be absent, and then so is the second sum
    n(x)    = x / sqrt(mean(x^2) + eps) * (1 + w)
    logits  = head n_final(x)
"""
from __future__ import annotations

import math

import numpy as np


def unit_rms(x, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    """The weight as it is stored: the norms inside a mixer."""
    return unit_rms(x, eps) * w


def rms_norm_about_one(x, w, eps):
    """A weight stored around nought: the norms of the layers and the last one."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * np.exp(-np.logaddexp(0.0, -z))


def heads_of(rows, heads):
    return rows.reshape(rows.shape[0], heads, -1)


# ---- rotations ---------------------------------------------------------------------------------------
def rotary_frequencies(rot):
    """What each of the dims/2 pairs advances by per position, and the factor on cos and sin."""
    dims, base = rot["dims"], float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def dim_of(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot, half: bool):
    """x [T, heads, n]: the first rot.dims entries of a head turn with the position, entry i with
    entry i + dims/2 (`half`) or entry 2i with 2i + 1; the rest pass."""
    dims = rot["dims"]
    f, mag = rotary_frequencies(rot)
    first, second = (slice(0, dims // 2), slice(dims // 2, dims)) if half else (slice(0, dims, 2), slice(1, dims, 2))
    out = np.array(x, np.float64)
    for p in range(x.shape[0]):
        c, s = np.cos(p * f) * mag, np.sin(p * f) * mag
        u, v = x[p, :, first], x[p, :, second]
        out[p, :, first] = u * c - v * s
        out[p, :, second] = v * c + u * s
    return out


# ---- retention ---------------------------------------------------------------------------------------
def decayed_state_walk(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv], decay [H]: S <- decay S + k v^T, o = S^T q."""
    T, H, d = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for a in range(H):
        S = np.zeros((d, v.shape[2]))
        for t in range(T):
            S = decay[a] * S + np.outer(k[t, a], v[t, a])
            out[t, a] = S.T @ q[t, a]
    return out


def retention(h, W, p, m, eps):
    """q and k turned, k times dim^(-1/2); every head's output of unit RMS, gated by a silu."""
    H = m["heads"]
    q, k, v = (heads_of(h @ W[p + n].T, H) for n in "qkv")
    q, k = rotate(q, m["rot"], True), rotate(k, m["rot"], True) * m["dim"] ** -0.5
    o = decayed_state_walk(q, k, v, np.asarray(m["decay"], np.float64))
    return (unit_rms(o, eps).reshape(len(h), -1) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- softmax attention --------------------------------------------------------------------------------
def causal_softmax(s):
    """s [T, T]: rows of weights over the keys up to the row's own."""
    s = np.where(np.tril(np.ones(s.shape, bool)), s, -np.inf)
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return e / e.sum(axis=1, keepdims=True)


def query_temperature(T, q_temp):
    """The factor on the queries of positions 0 .. T - 1."""
    if not q_temp:
        return np.ones(T)
    return np.array([1.0 + q_temp["coef"] * math.log(math.floor((p + 1) / q_temp["every"]) + 1.0) for p in range(T)])


def attention_keys(h, W, p, m, eps):
    """What a layer with keys of its own leaves for itself and for the layers that read it."""
    G = m["kv_heads"]
    return rms_norm(heads_of(h @ W[p + "k"].T, G), W[p + "k.norm"], eps), heads_of(h @ W[p + "v"].T, G)


def attention(h, W, p, m, eps, kv):
    """kv = (k [T, G, d], v [T, G, dv]) of this layer or of the one it reads."""
    H, G, T = m["heads"], m["kv_heads"], len(h)
    k, v = kv
    q = rms_norm(heads_of(h @ W[p + "q"].T, H), W[p + "q.norm"], eps) * query_temperature(T, m.get("q_temp"))[:, None, None]
    out = np.stack([causal_softmax(q[:, a] @ k[:, a // (H // G)].T * m["scale"]) @ v[:, a // (H // G)] for a in range(H)], axis=1)
    return out.reshape(T, -1) @ W[p + "o"].T


def latent_attention(h, W, p, m, eps):
    """Keys [W_uk c | rotated part shared by the heads] and values W_uv c out of one normed latent c."""
    H, d, r, T = m["heads"], m["dim"], m["kv_rank"], len(h)
    q = heads_of(h @ W[p + "q"].T, H)
    low = h @ W[p + "dkv"].T
    c = rms_norm(low[:, :r], W[p + "dkv.norm"], eps)
    k_rot = rotate(low[:, None, r:], m["rot"], False)[:, 0]
    q_rot = rotate(q[..., d:], m["rot"], False)
    k, v = heads_of(c @ W[p + "uk"].T, H), heads_of(c @ W[p + "uv"].T, H)
    out = np.stack([causal_softmax((q[:, a, :d] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"]) @ v[:, a] for a in range(H)], axis=1)
    return out.reshape(T, -1) @ W[p + "o"].T


# ---- feed-forward -------------------------------------------------------------------------------------
def gated(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def router_logits(h, W, p):
    return h @ W[p + "router"].T


def router_scores(h, W, p):
    z = router_logits(h, W, p)
    e = np.exp(z - z.max(axis=1, keepdims=True))
    return e / e.sum(axis=1, keepdims=True)


def routed_experts(h, W, p, mlp):
    """The largest scores of a softmax over all experts weigh their experts as they are."""
    s = router_scores(h, W, p)
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e in np.argsort(-s[t], kind="stable")[:mlp["router"]["top"]]:
            out[t] += s[t, e] * gated(h[t:t + 1], W, f"{p}e{e}.")[0]
    return out


def router_margins(h, W, p, mlp):
    """Per row, how far the last pick's logit lies above the first one not picked."""
    top, z = mlp["router"]["top"], -np.sort(-router_logits(h, W, p), axis=1)
    return z[:, top - 1] - z[:, top] if top < z.shape[1] else np.full(len(h), np.inf)


def feed_forward(h, W, p, mlp):
    return gated(h, W, p) if mlp["kind"] == "dense" else routed_experts(h, W, p, mlp)


def forward(config: dict, W: dict, tokens, return_layers: bool = False, margins: list | None = None, touch=lambda rows: rows):
    """logits [T, vocab] of one sequence from its first token; with return_layers also the rows after
    every layer; `margins` collects every routed layer's margins per row.  `touch`: what happens to
    the rows that each sublayer reads (nothing; a test that asks how far small errors spread disturbs
    them)."""
    W = {k: np.asarray(v, np.float64) for k, v in W.items()}
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    x = W["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    after, kept = [], {}
    for i, entry in enumerate(config["layers"]):
        p, m, h = f"l{i}.", entry["mixer"], touch(x)
        if entry["type"] == "retention":
            y = retention(h, W, p + "mix.", m, eps)
        elif entry["type"] == "latent_attention":
            y = latent_attention(h, W, p + "mix.", m, eps)
        else:
            if m.get("kv_from") is None:
                kept[i] = attention_keys(h, W, p + "mix.", m, eps)
            y = attention(h, W, p + "mix.", m, eps, kept[i if m.get("kv_from") is None else m["kv_from"]])
        x = x + mult * rms_norm_about_one(y, W[p + "norm1"], eps)
        if entry.get("mlp"):
            h = touch(x)
            if margins is not None and entry["mlp"]["kind"] == "moe":
                margins.append(router_margins(h, W, p + "mlp.", entry["mlp"]))
            x = x + mult * rms_norm_about_one(feed_forward(h, W, p + "mlp.", entry["mlp"]), W[p + "norm2"], eps)
        after.append(x)
    logits = rms_norm_about_one(x, W["final.norm"], eps) @ W["head"].T
    return (logits, np.stack(after)) if return_layers else logits
