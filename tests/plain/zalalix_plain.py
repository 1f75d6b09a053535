"""The Zalalix decoder as a plain function of a whole sequence, in double precision: one function
per mechanism, no cache, no batching, no kernels.  What the engine computes is held against this.

Notation: h [T, D] rows of one sequence in order; W a dict of arrays by tensor name; weights are
stored [out, in] and applied as W x; positions count from 0.

    x       = scale_e embed[token]
    layer   : x = x + n1b(mixer(n1(x)));  x = x + n2b(ff(n2(x)))      ff may be absent, and then so is the second sum
    n(x)    = x / sqrt(mean(x^2) + eps) * w
    logits  = head n_final(x)
"""
from __future__ import annotations

import math

import numpy as np


def unit_rms(x, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def silu(z):
    return z * sigmoid(z)


# ---- linear attention: a matrix state per head, S <- decay S + k v^T, o = S^T q --------------------
def decayed_state_walk(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv]; decay [T, H, d]: the factor on the state's row of each key entry."""
    T, H, d = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for a in range(H):
        S = np.zeros((d, v.shape[2]))
        for t in range(T):
            S = decay[t, a][:, None] * S + np.outer(k[t, a], v[t, a])
            out[t, a] = S.T @ q[t, a]
    return out


def heads_of(rows, heads):
    return rows.reshape(rows.shape[0], heads, -1)


def fixed_decays(m, T):
    return np.broadcast_to(np.asarray(m["decay"], np.float64)[None, :, None], (T, m["heads"], m["dim"]))


def lightning(h, W, p, m, eps):
    """q, k and v pass a silu; the heads' outputs are normed together, then gated by a sigmoid."""
    H = m["heads"]
    q, k, v = (heads_of(silu(h @ W[p + n].T), H) for n in "qkv")
    o = decayed_state_walk(q, k, v, fixed_decays(m, len(h))).reshape(len(h), -1)
    return (rms_norm(o, W[p + "norm"], eps) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def retention(h, W, p, m, eps):
    """k times dim^(-1/2); every head's output is made of unit RMS, then gated by a silu."""
    H = m["heads"]
    q, k, v = (heads_of(h @ W[p + n].T, H) for n in "qkv")
    o = decayed_state_walk(q, k * m["dim"] ** -0.5, v, fixed_decays(m, len(h)))
    return (unit_rms(o, eps).reshape(len(h), -1) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def channel_decays(h, W, p, m):
    """sigmoid(z)^(1/tau) per key channel, z through a product of low rank."""
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    return heads_of(np.exp(-np.logaddexp(0.0, -z) / m["tau"]), m["heads"])


def gated_linear_attention(h, W, p, m, eps):
    H = m["heads"]
    q, k, v = (heads_of(h @ W[p + n].T, H) for n in "qkv")
    o = decayed_state_walk(q * m["dim"] ** -0.5, k, v, channel_decays(h, W, p, m))
    return (rms_norm(o, W[p + "norm"], eps).reshape(len(h), -1) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- softmax attention ------------------------------------------------------------------------------
def rotary_frequencies(rot):
    """What each of the dims/2 pairs advances by per position: base^(-2i/dims); with scaling, pairs
    of long wavelength are slowed down by `factor`, pairs of short wavelength keep their pace, and
    between the two limits the two are blended."""
    dims = rot["dims"]
    out = []
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate(x, rot, positions=None):
    """x [T, heads, n]: entries 2i and 2i + 1 of a head's first rot.dims turn together; the rest pass."""
    f = rotary_frequencies(rot)
    dims = rot["dims"]
    out = np.array(x, np.float64)
    for t, p in enumerate(range(x.shape[0]) if positions is None else positions):
        c, s = np.cos(p * f), np.sin(p * f)
        u, v = x[t, :, 0:dims:2], x[t, :, 1:dims:2]
        out[t, :, 0:dims:2] = u * c - v * s
        out[t, :, 1:dims:2] = v * c + u * s
    return out


def sees(i, j, mask):
    return (j <= i) & ((i - j < mask["size"]) | (j < mask["keep_first"]))


def capped(s, cap):
    return cap * np.tanh(s / cap)


def softmax_attention(q, k, v, scale, cap, mask):
    """q [T, H, d], k [T, G, d], v [T, G, dv]: query head a reads KV head a // (H / G); the
    denominator holds one more term, exp(0), that has no value."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        keys = np.flatnonzero(sees(i, np.arange(T), mask))
        for a in range(H):
            g = a // (H // G)
            s = capped(k[keys, g] @ q[i, a] * scale, cap)
            top = max(s.max(), 0.0)
            e = np.exp(s - top)
            out[i, a] = e @ v[keys, g] / (e.sum() + math.exp(-top))
    return out


def windowed_attention(h, W, p, m, eps):
    """Biases; q and k RMS-normed over all their heads at once, then turned; one gate a head."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = len(h)
    q = rms_norm(h @ W[p + "q"].T + W[p + "q.b"], W[p + "q.norm"], eps).reshape(T, H, d)
    k = rms_norm(h @ W[p + "k"].T + W[p + "k.b"], W[p + "k.norm"], eps).reshape(T, G, d)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).reshape(T, G, dv)
    o = softmax_attention(rotate(q, m["rot"]), rotate(k, m["rot"]), v, m["scale"], m["softcap"], m["mask"])
    o = o * sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ W[p + "o"].T + W[p + "o.b"]


def parallel(h, W, p, m, eps):
    """Two mixers of the same rows, summed with a factor each."""
    left = windowed_attention(h, W, p + "left.", m["left"], eps)
    right = gated_linear_attention(h, W, p + "right.", m["right"], eps)
    return m["left_scale"] * left + m["right_scale"] * right


MIXERS = {"lightning": lightning, "retention": retention, "parallel": parallel}


def dense(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def forward(config: dict, W: dict, tokens, return_layers: bool = False, touch=lambda rows: rows):
    """logits [T, vocab] of one sequence from its first token; with return_layers also the rows
    after every layer.  `touch`: what happens to the rows that each sublayer reads (nothing; a test
    that asks how far small errors spread disturbs them)."""
    W = {k: np.asarray(v, np.float64) for k, v in W.items()}
    eps = config["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    after = []
    for i, entry in enumerate(config["layers"]):
        p = f"l{i}."
        y = MIXERS[entry["type"]](touch(rms_norm(x, W[p + "norm1"], eps)), W, p + "mix.", entry["mixer"], eps)
        x = x + rms_norm(y, W[p + "norm1b"], eps)
        if entry.get("mlp"):
            y = dense(touch(rms_norm(x, W[p + "norm2"], eps)), W, p + "mlp.")
            x = x + rms_norm(y, W[p + "norm2b"], eps)
        after.append(x)
    logits = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    return (logits, np.stack(after)) if return_layers else logits
