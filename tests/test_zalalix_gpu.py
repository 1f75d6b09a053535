"""Zalalix in the engine against the plain model of tests/plain/zalalix_plain.py: every mechanism
alone, prompts against token-by-token decoding, prompts cut into portions, batches of unequal
requests, slots and pages that are used again, one key that the asking token rests on far back, at page
borders, just inside and just outside the window and the kept first tokens, in prompts and decoded,
long decoding through recorded steps, and greedy generation through the entry points.

The configurations are those of tests/zalalix_tiny.py; the plain model computes a whole sequence
from scratch in double precision, so every schedule has one truth: the function of the sequence."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import zalalix_tiny as zt

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]


def tokens_for(cfg, n, seed):
    rng = np.random.default_rng(seed)
    return [int(t) for t in rng.integers(0, cfg["vocab"], size=n)]


_MODELS, _TRUTH = {}, {}


def model_of(which, dtype, seed=0):
    key = (which, dtype, seed)
    if key not in _MODELS:
        cfg = zt.CONFIGS[which]
        w = zt.make_weights(cfg, seed)
        _MODELS[key] = (cfg, w, zt.load(cfg, w, dtype))
    return _MODELS[key]


def truth_of(which, seed, tokens):
    key = (which, seed, tuple(tokens))
    if key not in _TRUTH:
        cfg = zt.CONFIGS[which]
        _TRUTH[key] = zt.Truth(cfg, zt.make_weights(cfg, seed), tokens)
    return _TRUTH[key]


def new_session(model, max_tokens=4096, **kw):
    from picolm_amd.engine import Session
    return Session(model, max_tokens=max_tokens, **kw)


def run_whole(session, tokens):
    [slot] = session.begin(1)
    got = session.step([slot], [tokens], [list(range(len(tokens)))]).double().cpu().numpy()
    session.release([slot])
    return got


# ------------------------------------------------------------------------------ each mechanism alone
def one_layer(mixer, ff=None, width=48, **kw):
    return zt.config(61, width, [zt.layer(mixer, ff)], **kw)


def attention_alone(*args, softcap=8.0, width=48, right=None, **kw):
    """The softmax branch; the other branch's factor is nought unless it is given."""
    return one_layer(zt.parallel(zt.windowed(*args, softcap=softcap), right or zt.gla(1, 4, 6, 2.0, 2), 1.0, 0.5 if right else 0.0), width=width, **kw)


def gla_alone(*args, width=48, **kw):
    return one_layer(zt.parallel(zt.windowed(1, 1, 4, 6, 0.5, 9, 0, zt.rotation(2)), zt.gla(*args), 0.0, 1.0), width=width, **kw)


_Y = zt.slowed(4.0, 1.0, 3.0, 64)
ALONE = {
    "a window and kept tokens": attention_alone(6, 2, 20, 12, 0.25, 17, 3, zt.rotation(8, 500.0)),
    "a window and nothing kept": attention_alone(2, 1, 12, 20, 0.3, 30, 0, zt.rotation(12, 100.0)),
    "a window of one, one kept": attention_alone(3, 3, 10, 6, 0.4, 1, 1, zt.rotation(4)),
    "more kept than the window": attention_alone(2, 2, 14, 6, 0.4, 5, 21, zt.rotation(2, 2.0)),
    "a window longer than the sequence": attention_alone(4, 2, 12, 10, 0.3, 500, 7, zt.rotation(6)),
    "more kept than the sequence": attention_alone(4, 1, 12, 10, 0.3, 4, 300, zt.rotation(6)),
    "a window of a page, a page kept": attention_alone(2, 1, 12, 10, 0.3, 64, 64, zt.rotation(6)),
    "slowed rotation": attention_alone(3, 1, 16, 20, 0.4, 40, 4, zt.rotation(16, 500.0, _Y)),
    "slowed rotation, every pair": attention_alone(3, 1, 16, 20, 0.4, 40, 4, zt.rotation(16, 10.0, zt.slowed(3.0, 1.0, 2.0, 1))),
    "slowed rotation, no pair": attention_alone(3, 1, 16, 20, 0.4, 40, 4, zt.rotation(16, 10.0, zt.slowed(3.0, 1.0, 2.0, 10 ** 6))),
    "slowed rotation, limits that meet": attention_alone(3, 1, 16, 20, 0.4, 40, 4, zt.rotation(16, 50.0, zt.slowed(3.0, 2.0, 2.0, 90))),
    "a cap that always binds": attention_alone(4, 2, 12, 10, 2.0, 20, 2, zt.rotation(6), softcap=0.5),
    "a cap that never binds": attention_alone(4, 2, 12, 10, 0.3, 20, 2, zt.rotation(6), softcap=1e4),
    "odd head sizes": attention_alone(5, 1, 9, 7, 0.4, 12, 2, zt.rotation(6), width=45),
    "one head of 3": attention_alone(1, 1, 3, 1, 0.6, 9, 2, zt.rotation(2)),
    "heads of 300": attention_alone(2, 1, 300, 24, 0.06, 40, 5, zt.rotation(100), width=64),
    "values of 288": attention_alone(2, 1, 24, 288, 0.2, 40, 5, zt.rotation(12), width=64),
    # sizes that the matrix-core kernel takes in bfloat16
    "keys of 64 and values of 96": attention_alone(4, 2, 64, 96, 0.15, 33, 6, zt.rotation(32, 1000.0, _Y), softcap=20.0, width=64),
    "keys of 96 and values of 64, nothing kept": attention_alone(2, 1, 96, 64, 0.1, 31, 0, zt.rotation(96), softcap=20.0, width=64),
    "keys of 128 and values of 128, forty heads": attention_alone(40, 8, 128, 128, 0.1, 20, 40, zt.rotation(64), softcap=5.0, width=64),
    "keys of 64, a cap that always binds": attention_alone(4, 1, 64, 64, 2.0, 20, 2, zt.rotation(64), softcap=1.0, width=64),
    "decays per channel": gla_alone(3, 10, 14, 4.0, 6),
    "decays per channel, tau of one": gla_alone(2, 16, 6, 1.0, 3),
    "decays per channel, one head, a rank of one": gla_alone(1, 5, 3, 16.0, 1),
    "decays per channel, heads of 64 and 128": gla_alone(2, 64, 128, 16.0, 16, width=64),
    "decays per channel, keys of 200": gla_alone(2, 200, 40, 8.0, 24, width=64),
    "decays per channel, a rank above the width": gla_alone(2, 20, 12, 2.0, 70),
    "lightning": one_layer(zt.lightning(14, 10, [0.5, 0.98, 0.999])),
    "lightning, one head": one_layer(zt.lightning(5, 9, [0.9])),
    "lightning, decays of nought and one": one_layer(zt.lightning(12, 12, [0.0, 1.0])),
    "lightning, heads of 128": one_layer(zt.lightning(128, 128, [0.9, 0.9995]), width=64),
    "lightning, keys of 256": one_layer(zt.lightning(256, 17, [0.99]), width=64),
    "lightning, 1,100 columns normed together": one_layer(zt.lightning(16, 220, [0.5, 0.8, 0.9, 0.99, 1.0]), width=64),
    "retention": one_layer(zt.retention(12, 20, [0.9, 0.995])),
    "retention, decays of nought and one": one_layer(zt.retention(7, 3, [1.0, 0.0, 0.5])),
    "retention, heads of 64": one_layer(zt.retention(64, 64, [0.9375, 0.9995]), width=64),
    "retention, keys of 200 and values of 1": one_layer(zt.retention(200, 1, [0.9]), width=64),
    "both branches": one_layer(zt.parallel(zt.windowed(4, 2, 12, 10, 0.3, 20, 3, zt.rotation(6)), zt.gla(3, 8, 14, 4.0, 5), 1.4, -0.6)),
    "both branches, heads of 64": one_layer(zt.parallel(zt.windowed(4, 2, 64, 64, 0.15, 20, 3, zt.rotation(32)), zt.gla(2, 64, 96, 4.0, 8)), width=64),
    "both branches, one branch's factor negative": one_layer(zt.parallel(zt.windowed(4, 2, 12, 10, 0.3, 20, 3, zt.rotation(6)), zt.gla(3, 8, 14, 4.0, 5), -1.0, 1.0)),
    "a feed-forward": one_layer(zt.retention(12, 20, [0.9, 0.995]), 40),
    "a feed-forward of 13 in a width of 45": one_layer(zt.retention(12, 20, [0.9, 0.995]), 13, width=45),
    "a feed-forward behind both branches": one_layer(zt.parallel(zt.windowed(4, 2, 12, 10, 0.3, 20, 3, zt.rotation(6)), zt.gla(3, 8, 14, 4.0, 5)), 72),
    "the embedding's factor": one_layer(zt.lightning(14, 10, [0.5]), 24, scale=0.01),
    "eps": one_layer(zt.parallel(zt.windowed(4, 2, 12, 10, 0.3, 20, 3, zt.rotation(6)), zt.gla(3, 8, 14, 4.0, 5)), 24, eps=0.3),
    "eps in retention": one_layer(zt.retention(12, 20, [0.9, 0.995]), 24, eps=0.3),
    "eps in lightning": one_layer(zt.lightning(12, 20, [0.9, 0.995]), 24, eps=0.3),
    "a width above what a workgroup keeps in registers": one_layer(zt.retention(8, 8, [0.9]), 16, width=2104),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", list(ALONE))
def test_each_mechanism_alone(what, dtype):
    cfg = ALONE[what]
    w = zt.make_weights(cfg, 11)
    tokens = tokens_for(cfg, 70, 3)            # past a page's end
    want = zt.Truth(cfg, w, tokens)
    s = new_session(zt.load(cfg, w, dtype), 256)
    assert zt.near(run_whole(s, tokens), want, slice(None), dtype)
    # and the same decoded token by token
    [slot] = s.begin(1)
    for i, t in enumerate(tokens):
        got = s.step([slot], [[t]]).double().cpu().numpy()
        assert zt.near(got, want, i, dtype), (what, "token", i)
    s.release([slot])


# what a configuration may leave out: no mask, no cap, no rotation (the plain model takes ones that change nothing)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim", [12, 64])
def test_attention_without_mask_cap_and_rotation(dim, dtype):
    cfg = attention_alone(4, 2, dim, dim, dim ** -0.5, 10 ** 6, 0, zt.rotation(2, 1.0000001), softcap=1e9, width=64)
    w = zt.make_weights(cfg, 11)
    bare = copy.deepcopy(cfg)
    left = bare["layers"][0]["mixer"]["left"]
    for key in ("mask", "softcap", "rot", "scale"):
        del left[key]
    tokens = tokens_for(cfg, 70, 3)
    from plain import zalalix_plain as P
    turned, P.rotate = P.rotate, lambda x, rot, positions=None: np.array(x)
    try:
        want = zt.Truth(cfg, w, tokens)
        want.limits(dtype)
    finally:
        P.rotate = turned
    s = new_session(zt.load(bare, w, dtype), 256)
    assert zt.near(run_whole(s, tokens), want, slice(None), dtype)


# ------------------------------------------------------------------------------ prompts, decoding, portions
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_prompt_decoding_and_portions(which, dtype):
    cfg, w, model = model_of(which, dtype)
    tokens = tokens_for(cfg, 150, 1)
    want = truth_of(which, 0, tokens)
    s = new_session(model, 1024)
    assert zt.near(run_whole(s, tokens), want, slice(None), dtype)
    # most of it at once, the rest one by one (past the page border at 128)
    [slot] = s.begin(1)
    got = s.step([slot], [tokens[:101]], [[0, 1, 2, 63, 64, 100]]).double().cpu().numpy()
    assert zt.near(got, want, [0, 1, 2, 63, 64, 100], dtype)
    for i in range(101, 150):
        got = s.step([slot], [[tokens[i]]]).double().cpu().numpy()
        assert zt.near(got, want, i, dtype), ("decoded", i)
    s.release([slot])
    # portions of several sizes, down to two tokens and one, every row wanted
    for sizes in ([2, 2, 3, 57, 1, 64, 21], [64, 64, 22], [1, 1, 2, 146], [149, 1], [36, 37, 38, 39]):
        assert sum(sizes) == 150
        [slot] = s.begin(1)
        at = 0
        for n in sizes:
            got = s.step([slot], [tokens[at:at + n]], [list(range(n))]).double().cpu().numpy()
            assert zt.near(got, want, slice(at, at + n), dtype), (sizes, "portion at", at)
            at += n
        s.release([slot])


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_equal_the_whole_prompt_beyond_rounding(dtype):
    """How a prompt is cut does not show in the logits: against each other, not only against the
    plain model, and much closer than the limit that bfloat16 needs there."""
    cfg, w, model = model_of("A", dtype)
    tokens = tokens_for(cfg, 131, 5)
    s = new_session(model, 1024)
    whole = run_whole(s, tokens)
    [slot] = s.begin(1)
    parts, at = [], 0
    for n in (2, 63, 2, 61, 3):
        parts.append(s.step([slot], [tokens[at:at + n]], [list(range(n))]).double().cpu().numpy())
        at += n
    s.release([slot])
    assert zt.distance(np.concatenate(parts), whole) <= (2e-5 if dtype == "float32" else 0.03)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "B"])
def test_a_long_prompt(which, dtype):
    """Several pages and several tiles of queries, prompts that the states are walked in chunks for, the
    last of them short; whole, in portions, and beside short requests in a batch, then decoded on."""
    cfg, w, model = model_of(which, dtype)
    tokens = tokens_for(cfg, 405, 8)
    want = truth_of(which, 0, tokens)
    s = new_session(model, 2048)
    assert zt.near(run_whole(s, tokens[:401]), want, slice(0, 401), dtype)
    [slot] = s.begin(1)
    rows = [0, 63, 64, 100]
    got = s.step([slot], [tokens[:101]], [rows]).double().cpu().numpy()
    assert zt.near(got, want, rows, dtype)
    got = s.step([slot], [tokens[101:401]], [list(range(300))]).double().cpu().numpy()
    assert zt.near(got, want, slice(101, 401), dtype)
    for i in range(401, 405):
        got = s.step([slot], [[tokens[i]]]).double().cpu().numpy()
        assert zt.near(got, want, i, dtype), ("decoded", i)
    s.release([slot])
    others = [tokens_for(cfg, n, 30 + n) for n in (10, 257)]
    slots = s.begin(3)
    got = s.step(slots, [tokens[:400]] + others).double().cpu().numpy()
    assert zt.near(got[0], want, 399, dtype)
    for i, q in enumerate(others):
        assert zt.near(got[1 + i], truth_of(which, 0, q), len(q) - 1, dtype), ("beside the long one", i)
    got = s.step(slots[:1], [[tokens[400]]]).double().cpu().numpy()
    assert zt.near(got, want, 400, dtype)
    s.release(slots)


# strong decays, weak ones, and channels that forget everything at once, over a prompt long enough to be walked in chunks
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,dim,vdim", [("gla", 20, 12), ("gla", 64, 128), ("gla", 128, 64), ("retention", 64, 96), ("lightning", 128, 128),
                                           ("retention", 40, 24), ("lightning", 200, 72)])
def test_states_over_a_long_prompt_of_uneven_decays(kind, dim, vdim, dtype):
    decays = [1.0, 0.0, 0.3, 0.999]
    if kind == "gla":
        cfg = gla_alone(3, dim, vdim, 1.0, 4, width=64)
    else:
        cfg = one_layer((zt.retention if kind == "retention" else zt.lightning)(dim, vdim, decays), width=64)
    w = zt.make_weights(cfg, 4)
    if kind == "gla":
        # of every eight key channels: one that keeps everything, one that forgets all but everything, others between
        b = torch.tensor([40.0, -90.0, 6.0, 3.0, 0.0, -3.0, -12.0, 9.0]).repeat(3 * dim // 8 + 1)[:3 * dim]
        w["l0.mix.right.a2.b"] = b.to(torch.bfloat16)
    tokens = tokens_for(cfg, 330, 9)
    want = zt.Truth(cfg, w, tokens)
    s = new_session(zt.load(cfg, w, dtype), 1024)
    assert zt.near(run_whole(s, tokens), want, slice(None), dtype)
    [slot] = s.begin(1)
    at = 0
    for n in (3, 259, 65, 1, 2):
        got = s.step([slot], [tokens[at:at + n]], [list(range(n))]).double().cpu().numpy()
        assert zt.near(got, want, slice(at, at + n), dtype), ("portion at", at)
        at += n
    s.release([slot])


# ------------------------------------------------------------------------------ batches
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "C"])
def test_a_batch_of_unequal_requests_equals_each_alone(which, dtype):
    cfg, w, model = model_of(which, dtype)
    lens, n_dec = [1, 2, 65, 37, 64, 130], 5
    seqs = [tokens_for(cfg, n + n_dec, 20 + i) for i, n in enumerate(lens)]
    truth = [truth_of(which, 0, q) for q in seqs]
    s = new_session(model, 2048)
    slots = s.begin(len(seqs))
    got = s.step(slots, [q[:n] for q, n in zip(seqs, lens)], [list(range(n)) for n in lens]).double().cpu().numpy()
    at = 0
    for i, n in enumerate(lens):
        assert zt.near(got[at:at + n], truth[i], slice(0, n), dtype), ("prompt", i)
        at += n
    # and against each alone, much closer than the plain model is in bfloat16: what else is in the batch does not show
    alone = new_session(model, 512)
    at = 0
    for i, n in enumerate(lens):
        assert zt.distance(got[at:at + n], run_whole(alone, seqs[i][:n])) <= (2e-5 if dtype == "float32" else 0.03), ("alone", i)
        at += n
    # the shorter ones end earlier: after two steps the first two leave the batch
    live = list(range(len(seqs)))
    for j in range(n_dec):
        if j == 2:
            s.release([slots[0], slots[1]])
            live = live[2:]
        got = s.step([slots[i] for i in live], [[seqs[i][lens[i] + j]] for i in live]).double().cpu().numpy()
        for row, i in enumerate(live):
            assert zt.near(got[row], truth[i], lens[i] + j, dtype), ("step", j, "sequence", i)
    s.release([slots[i] for i in live])


@pytest.mark.parametrize("dtype", DTYPES)
def test_slots_and_pages_that_are_used_again(dtype):
    """A page's old keys are not seen and a slot's old state is gone: sequences run one after another
    through a session that has room for little more than one of them."""
    cfg, w, model = model_of("A", dtype)
    s = new_session(model, 256, n_slots=2)
    for k, n in enumerate([130, 5, 70, 130, 1, 64]):
        tokens = tokens_for(cfg, n, 40 + k)
        want = truth_of("A", 0, tokens)
        [slot] = s.begin(1)
        cut = max(1, n - 3)
        rows = [0, cut - 1]
        got = s.step([slot], [tokens[:cut]], [rows]).double().cpu().numpy()
        assert zt.near(got, want, rows, dtype), ("prompt", k)
        for i in range(cut, n):
            got = s.step([slot], [[tokens[i]]]).double().cpu().numpy()
            assert zt.near(got, want, i, dtype), ("sequence", k, "token", i)
        s.release([slot])
    # two sequences that swap slots between uses
    a, b = tokens_for(cfg, 40, 90), tokens_for(cfg, 66, 91)
    for order in ((a, b), (b, a)):
        slots = s.begin(2)
        got = s.step(slots, list(order)).double().cpu().numpy()
        for i, q in enumerate(order):
            assert zt.near(got[i], truth_of("A", 0, q), len(q) - 1, dtype)
        s.release(slots)


# ------------------------------------------------------------------------------ far keys, page borders, the window's edges
def lookup_model(dim, size, keep, width=64):
    """One parallel layer whose attention looks a token's partner up (the other branch's factor is
    nought).  Token t + 700 has the first half of token t's embedding.  Keys read the first half of the
    width and queries are the keys' rows, so the score of two tokens with the same first half is as high
    as a token's with itself and far above the chance products of hundreds of other keys; what the
    partner contributes differs from the asking token's own contribution through the second half of the
    width (the values read it).  Few entries are turned, so that the position hardly weakens the match.
    So the asking token's output rests on its partner wherever the partner stands, if it is seen."""
    half, heads = width // 2, 2
    cfg = zt.config(1400, width, [zt.layer(zt.parallel(
        zt.windowed(heads, 1, dim, dim if dim == 64 else 16, 30.0 / dim, size, keep, zt.rotation(4, 10000.0, zt.slowed(4.0, 1.0, 3.0, 64)), 60.0),
        zt.gla(1, 4, 6, 2.0, 2), 1.0, 0.0))])
    w = zt.make_weights(cfg, 5)
    w["embed"][700:, :half] = w["embed"][:700, :half]
    for n in ("l0.norm1", "l0.mix.left.q.norm", "l0.mix.left.k.norm"):
        w[n] = torch.ones_like(w[n])
    p = "l0.mix.left."
    gen = torch.Generator().manual_seed(2)
    keys = torch.randn(dim, width, generator=gen, dtype=torch.float64) / half ** 0.5
    keys[:, half:] = 0
    w[p + "k"] = keys.to(torch.bfloat16)
    w[p + "q"] = torch.cat([keys] * heads).to(torch.bfloat16)
    for n in ("q.b", "k.b", "v.b", "o.b"):
        w[p + n] = (0.1 * w[p + n].double()).to(torch.bfloat16)
    w[p + "v"][:, :half] = 0
    w["l0.norm1b"] = (16.0 * w["l0.norm1b"].double()).to(torch.bfloat16)          # the branch outweighs the rows it is added to
    return cfg, w


def distinct_tokens(n, needle_at, vocab, seed):
    """n unrelated tokens, except that the last one's partner stands at `needle_at`."""
    rng = np.random.default_rng(seed)
    tokens = [int(t) for t in rng.permutation(vocab // 2)[:n]]
    tokens[needle_at] = tokens[-1] + vocab // 2
    return tokens


def without_the_partner(tokens, needle_at, vocab):
    other = list(tokens)
    other[needle_at] = next(t for t in range(vocab // 2) if t not in tokens)
    return other


_FAR = {}


def asking_sequence(key, cfg, w, n, needle_at, seed, seen=True):
    """n tokens whose last one's partner stands at `needle_at`, the plain model's logits of the last
    token, and a check that the test can tell: with the partner replaced by an unrelated token the
    logits differ by far more than rounding if the partner is seen (tokens are drawn again until
    they do), and not at all if it lies behind the window (while they would if everything were seen)."""
    if key in _FAR:
        return _FAR[key]
    from plain import zalalix_plain as P
    arrays = zt.as_arrays(w)
    last = lambda c, t: P.forward(c, arrays, t)[-1]
    while True:
        tokens = distinct_tokens(n, needle_at, cfg["vocab"], seed)
        other = without_the_partner(tokens, needle_at, cfg["vocab"])
        want, missed = last(cfg, tokens), last(cfg, other)
        if not seen:
            assert zt.distance(missed, want) < 1e-9, "the key must not count"
            whole = copy.deepcopy(cfg)
            whole["layers"][0]["mixer"]["left"]["mask"]["size"] = n
            counts = zt.distance(last(whole, other), last(whole, tokens))
        else:
            counts = zt.distance(missed, want) if needle_at != n - 1 else 1.0
        if counts > 0.2:
            _FAR[key] = (tokens, want)
            return _FAR[key]
        seed += 1000


def ask_in_a_prompt_and_decoded(s, tokens, want, dtype, what):
    [slot] = s.begin(1)
    got = s.step([slot], [tokens]).double().cpu().numpy()
    assert zt.distance(got, want) <= zt.LIMIT[dtype], ("prompt",) + what
    s.release([slot])
    [slot] = s.begin(1)
    s.step([slot], [tokens[:-1]], [[]])
    got = s.step([slot], [tokens[-1:]]).double().cpu().numpy()
    assert zt.distance(got, want) <= zt.LIMIT[dtype], ("decoded",) + what
    s.release([slot])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim", [20, 64])
def test_one_far_key_among_hundreds(dim, dtype):
    """The asking token is the last; the key it asks for lies hundreds back, at the first places of
    the sequence, and just before and after page borders.  Both in a prompt and decoded.  (Keys of 64
    go through the matrix-core kernel in bfloat16, the others through the vector ALU.)"""
    cfg, w = lookup_model(dim, 1000, 0)
    s = new_session(zt.load(cfg, w, dtype), 2048)
    n = 500
    for needle_at in (0, 1, 63, 64, 65, 128, 383, 498):
        tokens, want = asking_sequence((dim, needle_at), cfg, w, n, needle_at, needle_at)
        ask_in_a_prompt_and_decoded(s, tokens, want, dtype, (needle_at,))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,keep,dim", [(70, 5, 20), (64, 1, 20), (1, 3, 20), (2, 70, 20), (33, 4, 64), (100, 70, 64), (190, 0, 64), (65, 130, 64)])
def test_a_key_just_inside_and_just_outside_the_window_and_the_kept_tokens(size, keep, dim, dtype):
    """The partner of the last token stands at the oldest place of the window and the place before it,
    and at the last kept first token and the place after it: seen, the logits rest on it; not seen,
    they are what they are without it."""
    cfg, w = lookup_model(dim, size, keep)
    s = new_session(zt.load(cfg, w, dtype), 1024)
    for n in (size + keep + 40, 3 * size + 2 * keep + 7, 400):
        first = n - size                                   # the window's oldest place
        for needle_at, seen in ((first, True), (first - 1, False), (keep - 1, True), (0, keep > 0), (keep, False), (n - 2, size > 1 or keep > n - 2)):
            if needle_at < 0 or (not seen and needle_at < keep) or (needle_at >= first) != seen and needle_at >= keep:
                continue
            tokens, want = asking_sequence((size, keep, dim, n, needle_at), cfg, w, n, needle_at, n + needle_at, seen)
            ask_in_a_prompt_and_decoded(s, tokens, want, dtype, (n, needle_at, seen))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,keep,dim", [(70, 3, 20), (37, 66, 64)])
def test_a_window_passes_over_decoded_tokens(size, keep, dim, dtype):
    """A short prompt, then single tokens until the asking one, in a batch with a sequence that
    started elsewhere: the partner was decoded at the window's oldest place (seen) or just before it
    (not seen), or is a kept first token, of the prompt or decoded, or the one after those."""
    cfg, w = lookup_model(dim, size, keep)
    s = new_session(zt.load(cfg, w, dtype), 1024)
    beside = distinct_tokens(400, 3, cfg["vocab"], 77)
    n = 2 * size + keep + 9
    for needle_at, seen in ((n - size, True), (n - size - 1, False), (1, True), (keep - 1, True), (keep, False)):
        tokens, want = asking_sequence(("decoded", size, keep, dim, needle_at), cfg, w, n, needle_at, needle_at, seen)
        slots = s.begin(2)
        s.step(slots, [tokens[:8], beside[:400 - (n - 8)]], [[], []])
        for i in range(8, n):
            got = s.step(slots, [[tokens[i]], [beside[400 - n + i]]]).double().cpu().numpy()
        assert zt.distance(got[0], want) <= zt.LIMIT[dtype], (needle_at, seen)
        s.release(slots)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["gla", "retention", "lightning"])
def test_a_far_token_in_a_state_that_keeps(kind, dtype):
    """States whose decays are all but one: what a token wrote hundreds of tokens ago, in the first chunk
    of a prompt, at a chunk's edge, or in an earlier step, is in the output of the last."""
    dim, n = 96, 300
    if kind == "gla":
        cfg = gla_alone(1, dim, 24, 2.0, 3, width=64)
    else:
        cfg = one_layer((zt.retention if kind == "retention" else zt.lightning)(dim, 24, [1.0]), width=64)
    w = zt.make_weights(cfg, 6)
    p = "l0.mix.right." if kind == "gla" else "l0.mix."
    if kind == "gla":
        w[p + "a2.b"] = torch.full_like(w[p + "a2.b"], 40.0)
    w[p + "q"] = w[p + "k"].clone()
    # one rare token with a strong key and value of its own direction: token 60 is unlike the others
    w["embed"][60] = 0
    w["embed"][60, :8] = 3.0
    w["l0.norm1"] = torch.ones_like(w["l0.norm1"])
    w[p + "k"][:, :8] = (4.0 * w[p + "k"][:, :8].double()).to(torch.bfloat16)
    w[p + "v"][:, :8] = (4.0 * w[p + "v"][:, :8].double()).to(torch.bfloat16)
    w[p + "q"] = w[p + "k"].clone()
    w["embed"][:60, :8] = (0.2 * w["embed"][:60, :8].double()).to(torch.bfloat16)
    w["embed"][59, :8] = 3.0                  # the token that asks
    w["l0.norm1b"] = (8.0 * w["l0.norm1b"].double()).to(torch.bfloat16)
    s = new_session(zt.load(cfg, w, dtype), 1024)
    rng = np.random.default_rng(1)
    for at in (0, 1, 63, 64, 65, 255, 256, 298):
        tokens = [int(t) for t in rng.integers(0, 59, size=n)]
        tokens[-1] = 59
        without = list(tokens)
        tokens[at] = 60
        want = zt.plain_logits(cfg, w, tokens)[-1]
        assert zt.distance(zt.plain_logits(cfg, w, without)[-1], want) > 0.2, "the token must count"
        ask_in_a_prompt_and_decoded(s, tokens, want, dtype, (kind, at))


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_tokens_of_a_sequence(dtype):
    """Sequences of one, two and three tokens, alone and in one batch; windows of one and two."""
    cfg, w, model = model_of("C", dtype)
    s = new_session(model, 512)
    seqs = [tokens_for(cfg, n, 60 + n) for n in (1, 2, 3, 1)]
    for q in seqs:
        assert zt.near(run_whole(s, q), truth_of("C", 0, q), slice(None), dtype)
    slots = s.begin(len(seqs))
    got = s.step(slots, seqs).double().cpu().numpy()
    for i, q in enumerate(seqs):
        assert zt.near(got[i], truth_of("C", 0, q), len(q) - 1, dtype)
    s.release(slots)


# ------------------------------------------------------------------------------ long decoding
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "B"])
def test_long_decoding_through_recorded_steps(which, dtype):
    """Three sequences decoded 200 tokens, over page borders and past windows; from the second step of
    a shape on the engine replays its recording."""
    cfg, w, model = model_of(which, dtype)
    lens, n_dec = [3, 60, 120], 200
    seqs = [tokens_for(cfg, n + n_dec, 70 + i) for i, n in enumerate(lens)]
    truth = [truth_of(which, 0, q) for q in seqs]
    s = new_session(model, 2048)
    slots = s.begin(3)
    s.step(slots, [q[:n] for q, n in zip(seqs, lens)])
    for j in range(n_dec):
        got = s.step(slots, [[q[n + j]] for q, n in zip(seqs, lens)]).double().cpu().numpy()
        for i, n in enumerate(lens):
            assert zt.near(got[i], truth[i], n + j, dtype), ("step", j, "sequence", i)
    assert s.recorded_steps() >= 1
    s.release(slots)


@pytest.mark.parametrize("dtype", DTYPES)
def test_recorded_and_launched_steps_give_the_same_bits(dtype):
    cfg, w, model = model_of("A", dtype)
    seqs = [tokens_for(cfg, n + 12, 170 + i) for i, n in enumerate([5, 70])]
    rows = {}
    for graphs in (True, False):
        s = new_session(model, 1024, graphs=graphs)
        slots = s.begin(2)
        s.step(slots, [seqs[0][:5], seqs[1][:70]])
        rows[graphs] = [s.step(slots, [[seqs[0][5 + j]], [seqs[1][70 + j]]]).cpu().numpy().copy() for j in range(12)]
        s.release(slots)
    for a, b in zip(rows[True], rows[False]):
        assert np.array_equal(a, b)


# ------------------------------------------------------------------------------ the entry points
@pytest.fixture(scope="module")
def folder_a(tmp_path_factory):
    cfg = copy.deepcopy(zt.CONFIGS["A"])
    for l in cfg["layers"]:
        if l["type"] == "parallel":
            del l["mixer"]["right"]["rank"]               # the checkpoint's tensors say it
    return zt.write_folder(str(tmp_path_factory.mktemp("zalalix") / "a"), cfg, zt.make_weights(zt.CONFIGS["A"], 0))


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_entry_point(dtype, folder_a):
    import picolm_amd
    prompts = [tokens_for(zt.CONFIGS["A"], n, 50 + n) for n in (4, 9, 66)]
    got = picolm_amd.generate(folder_a, prompts, max_new_tokens=10, stop_ids=(), dtype=dtype)
    for p, r in zip(prompts, got):
        assert len(r.tokens) == 10 and r.finish == "length"
        seq = list(p)
        for k in range(10):
            lg = truth_of("A", 0, seq)[-1]
            top2 = np.sort(lg)[-2:]
            if top2[1] - top2[0] < 4 * zt.LIMIT[dtype] * lg.std():
                break                              # a near tie: either choice is right
            assert r.tokens[k] == int(np.argmax(lg)), (k, r.tokens)
            seq.append(r.tokens[k])


def test_trace_replay_and_command_line(folder_a, tmp_path):
    """bin/trace_run on a folder: a prompt, single tokens and a second request that joins later in a
    slot that was given back; bin/picolm generates from the same folder."""
    cfg = zt.CONFIGS["A"]
    a, b = tokens_for(cfg, 20, 1), tokens_for(cfg, 9, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[17:18], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[18:19], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[19:20], "want": [0]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "b", "tokens": b, "want": [8]}], "end": ["b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = str(tmp_path / "out")
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder_a, "--dtype", "float32", "--out", out,
                        "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                       timeout=300)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    ta, tb = truth_of("A", 0, a), truth_of("A", 0, b)
    read = lambda i: np.fromfile(os.path.join(out, f"{i}.f32"), dtype="<f4").reshape(-1, cfg["vocab"])
    assert zt.near(read(0), ta, [0, 16], "float32")
    assert zt.near(read(1), ta, 17, "float32")
    assert not os.path.exists(os.path.join(out, "2.f32"))
    assert zt.near(read(3), ta, 19, "float32")
    assert zt.near(read(4), tb, 8, "float32")
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "picolm"), folder_a, "-p", " ".join(map(str, b)), "-n", "4", "-t", "0",
                        "--dtype", "float32"], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert len(r.stdout.split()) == 4
    assert int(r.stdout.split()[0]) == int(np.argmax(tb[-1]))
