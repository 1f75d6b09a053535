"""Belorax in the engine against the plain model of tests/plain/belorax_plain.py: every mechanism alone,
prompts against token-by-token decoding, prompts cut into portions, batches of unequal requests, slots
and pages that are used again, one key that the asking token rests on far back, at page borders and at
the first places (kept by the asking layer or by an earlier one whose keys it reads, or held in a state),
in prompts and decoded, long decoding through recorded steps, and greedy generation through the entry
points.

The configurations are those of tests/belorax_tiny.py; the plain model computes a whole sequence
from scratch in double precision, so every schedule has one truth: the function of the sequence."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import belorax_tiny as bt

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]


def tokens_for(cfg, n, seed):
    rng = np.random.default_rng(seed)
    return [int(t) for t in rng.integers(0, cfg["vocab"], size=n)]


_MODELS, _TRUTH = {}, {}


def model_of(which, dtype, seed=0):
    key = (which, dtype, seed)
    if key not in _MODELS:
        cfg = bt.CONFIGS[which]
        w = bt.make_weights(cfg, seed)
        _MODELS[key] = (cfg, w, bt.load(cfg, w, dtype))
    return _MODELS[key]


def truth_of(which, seed, tokens):
    key = (which, seed, tuple(tokens))
    if key not in _TRUTH:
        cfg = bt.CONFIGS[which]
        _TRUTH[key] = bt.Truth(cfg, bt.make_weights(cfg, seed), tokens)
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
def one_layer(mixer, mlp=None, width=48, **kw):
    return bt.config(61, width, [bt.layer(mixer, mlp)], **kw)


def reading(mixer, width=48, **kw):
    """A layer that keeps keys, one of another kind, and two that read the first one's keys with other temperatures and scales."""
    m = mixer[1]
    reads = lambda scale, coef, every: bt.attention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale, coef, every, kv_from=0)
    return bt.config(61, width, [bt.layer(mixer), bt.layer(bt.retention(6, 4, [0.9], bt.rotation(4))), bt.layer(reads(0.7 * m["scale"], 0.0, 5)),
                                 bt.layer(reads(1.3 * m["scale"], 1.5, 9))], **kw)


_Y = bt.yarn(4.0, 64, 8.0, 2.0)
_ATTN = bt.attention(4, 2, 12, 10, 0.3)
ALONE = {
    "attention": one_layer(bt.attention(6, 2, 20, 12, 0.25)),
    "attention, a KV head a head": one_layer(bt.attention(3, 3, 10, 16, 0.4)),
    "attention, one head of 3": one_layer(bt.attention(1, 1, 3, 1, 0.6)),
    "attention, odd head sizes": one_layer(bt.attention(5, 1, 9, 7, 0.4), width=45),
    "attention, heads of 300": one_layer(bt.attention(2, 1, 300, 24, 0.06), width=64),
    "attention, values of 288": one_layer(bt.attention(2, 1, 24, 288, 0.2), width=64),
    "attention, a temperature of one token a step": one_layer(bt.attention(4, 2, 12, 10, 0.3, 2.0, 1)),
    "attention, a temperature that falls": one_layer(bt.attention(4, 2, 12, 10, 0.5, -0.2, 3)),
    "attention, a temperature that changes once": one_layer(bt.attention(4, 2, 12, 10, 0.3, 3.0, 36)),
    "attention, a temperature that never changes": one_layer(bt.attention(4, 2, 12, 10, 0.3, 3.0, 1000)),
    "attention, steps of two and a half tokens": one_layer(bt.attention(4, 2, 12, 10, 0.3, 1.0, 2.5)),
    "attention, no temperature": one_layer(bt.attention(4, 2, 12, 10, 0.3, 0.0, 8)),
    # sizes that the matrix-core kernel takes in bfloat16
    "attention, keys of 64 and values of 96": one_layer(bt.attention(4, 2, 64, 96, 0.15, 0.6, 7), width=64),
    "attention, keys of 96 and values of 64": one_layer(bt.attention(2, 1, 96, 64, 0.1, 0.6, 7), width=64),
    "attention, keys and values of 128, forty heads": one_layer(bt.attention(40, 8, 128, 128, 0.1, 0.6, 7), width=64),
    "read keys": reading(bt.attention(6, 2, 20, 12, 0.25, 0.8, 11)),
    "read keys, one head": reading(bt.attention(1, 1, 5, 40, 0.4, 0.8, 11)),
    "read keys of 64 and values of 128": reading(bt.attention(4, 2, 64, 128, 0.15, 0.8, 11), width=64),
    "read keys of 96 and values of 96": reading(bt.attention(8, 1, 96, 96, 0.12, 0.8, 11), width=64),
    "latent attention": one_layer(bt.latent(3, 12, 8, 20, 28, 0.4)),
    "latent attention, scaled rotation": one_layer(bt.latent(3, 12, 16, 20, 28, 0.4, 500.0, _Y)),
    "latent attention, a ramp that starts later": one_layer(bt.latent(3, 12, 16, 20, 28, 0.4, 500.0, bt.yarn(4.0, 80, 1.0, 0.25))),
    "latent attention, a ramp of one pair": one_layer(bt.latent(2, 8, 12, 6, 10, 0.4, 30.0, bt.yarn(16.0, 40, 2.0, 1.9))),
    "latent attention, a rotated part of two": one_layer(bt.latent(3, 14, 2, 6, 10, 0.4, 2.0, bt.yarn(2.0, 8, 4.0, 1.0))),
    "latent attention, one head, latents of 5": one_layer(bt.latent(1, 7, 4, 3, 5, 0.6)),
    "latent attention, keys of 64 over latents of 32": one_layer(bt.latent(4, 24, 32, 16, 32, 0.3, 1000.0, _Y)),
    "latent attention, keys of 96 over latents of 64": one_layer(bt.latent(4, 24, 32, 40, 64, 0.2, 1000.0, _Y)),
    "latent attention, keys of 128 over latents of 96, forty heads": one_layer(bt.latent(40, 8, 32, 12, 96, 0.3)),
    "latent attention, keys of 320": one_layer(bt.latent(2, 16, 32, 24, 288, 0.15)),
    "retention": one_layer(bt.retention(12, 20, [0.9, 0.995], bt.rotation(12, 100.0))),
    "retention, a part of a head turned": one_layer(bt.retention(20, 12, [0.9, 0.995, 0.7], bt.rotation(6, 30.0))),
    "retention, one pair turned": one_layer(bt.retention(9, 12, [0.95], bt.rotation(2))),
    "retention, decays of nought and one": one_layer(bt.retention(8, 3, [1.0, 0.0, 0.5], bt.rotation(8))),
    "retention, heads of 64": one_layer(bt.retention(64, 64, [0.9375, 0.9995], bt.rotation(64, 1000.0)), width=64),
    "retention, keys of 200 and values of 1": one_layer(bt.retention(200, 1, [0.9], bt.rotation(100)), width=64),
    "retention, keys of 256 and values of 130": one_layer(bt.retention(256, 130, [0.99], bt.rotation(256)), width=64),
    "retention, the keys' factor beside a large eps": one_layer(bt.retention(12, 20, [0.9, 0.995], bt.rotation(12)), eps=0.3),
    "a dense feed-forward": one_layer(_ATTN, bt.dense(40)),
    "a feed-forward of 13 in a width of 45": one_layer(_ATTN, bt.dense(13), width=45),
    "routed experts": one_layer(_ATTN, bt.moe(6, 2, 24)),
    "routed experts, their scores beside a large eps": one_layer(_ATTN, bt.moe(6, 2, 24), eps=0.3),
    "routed experts, one pick": one_layer(_ATTN, bt.moe(5, 1, 36), eps=0.1),
    "routed experts, every expert picked": one_layer(_ATTN, bt.moe(3, 3, 20), eps=0.1),
    "one routed expert": one_layer(_ATTN, bt.moe(1, 1, 20)),
    # in bfloat16 a prompt of 64 rows and more sorts its picks by expert for the matrix cores
    "routed experts, widths in multiples of 16": one_layer(_ATTN, bt.moe(6, 2, 32), eps=0.1),
    "routed experts, more experts than rows a tile": one_layer(_ATTN, bt.moe(40, 3, 48), eps=1e-3),
    "routed experts, widths that are no multiples of 8": one_layer(_ATTN, bt.moe(4, 2, 13), width=45),
    "the branches' factor": one_layer(_ATTN, bt.dense(24), mult=3.0),
    "the branches' factor, negative": one_layer(_ATTN, bt.dense(24), mult=-0.25),
    "a factor of one": one_layer(_ATTN, bt.dense(24), mult=1.0, scale=1.0),
    "the embedding's factor": one_layer(_ATTN, bt.dense(24), scale=12.0),
    "a width above what a workgroup keeps in registers": one_layer(bt.retention(8, 8, [0.9], bt.rotation(8)), bt.dense(16), width=2104),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", list(ALONE))
def test_each_mechanism_alone(what, dtype):
    cfg = ALONE[what]
    w = bt.make_weights(cfg, 11)
    tokens = tokens_for(cfg, 70, 3)            # past a page's end
    want = bt.Truth(cfg, w, tokens)
    s = new_session(bt.load(cfg, w, dtype), 256)
    assert bt.near(run_whole(s, tokens), want, slice(None), dtype)
    # and the same decoded token by token
    [slot] = s.begin(1)
    for i, t in enumerate(tokens):
        got = s.step([slot], [[t]]).double().cpu().numpy()
        assert bt.near(got, want, i, dtype), (what, "token", i)
    s.release([slot])


# what a configuration may leave out: a rotation, a temperature
@pytest.mark.parametrize("dtype", DTYPES)
def test_layers_without_rotation_and_temperature(dtype):
    cfg = bt.config(61, 48, [bt.layer(bt.retention(12, 20, [0.9, 0.995], bt.rotation(2))), bt.layer(bt.attention(4, 2, 12, 10, 0.3, 0.0, 1))])
    bare = copy.deepcopy(cfg)
    del bare["layers"][0]["mixer"]["rot"], bare["layers"][1]["mixer"]["q_temp"]
    w = bt.make_weights(cfg, 11)
    tokens = tokens_for(cfg, 70, 3)
    from plain import belorax_plain as P
    turned, P.rotate = P.rotate, lambda x, rot, half: np.array(x)
    try:
        want = bt.Truth(cfg, w, tokens)
        want.limits(dtype)
    finally:
        P.rotate = turned
    s = new_session(bt.load(bare, w, dtype), 256)
    assert bt.near(run_whole(s, tokens), want, slice(None), dtype)
    [slot] = s.begin(1)
    for i, t in enumerate(tokens):
        assert bt.near(s.step([slot], [[t]]).double().cpu().numpy(), want, i, dtype), ("token", i)
    s.release([slot])


# what the design does not use of the parts' new options
@pytest.mark.parametrize("dtype", DTYPES)
def test_retention_that_turns_neighbours(dtype):
    cfg = one_layer(bt.retention(20, 12, [0.9, 0.995], bt.rotation(14, 30.0)))
    w = bt.make_weights(cfg, 11)
    tokens = tokens_for(cfg, 70, 3)
    from picolm_amd.engine.builder import build_from_config_dict, parse_dtype
    from picolm_amd.parts.base import Runtime
    from picolm_amd.weights import TensorDict
    from plain import belorax_plain as P
    turned, P.rotate = P.rotate, lambda x, rot, half: turned(x, rot, False)
    try:
        want = bt.Truth(cfg, w, tokens)
        want.limits(dtype)
    finally:
        P.rotate = turned
    model = build_from_config_dict(cfg)
    model.blocks[0].mixer.position.style = "pairwise"
    model.load(TensorDict(w), Runtime(torch.device("cuda:0"), parse_dtype(dtype)))
    s = new_session(model, 256)
    assert bt.near(run_whole(s, tokens), want, slice(None), dtype)
    [slot] = s.begin(1)
    for i, t in enumerate(tokens):
        assert bt.near(s.step([slot], [[t]]).double().cpu().numpy(), want, i, dtype), ("token", i)
    s.release([slot])


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_block_of_output_norms_beside_a_pre_norm_block_and_read_keys_behind_a_norm_over_all_heads(dtype):
    """Parts put together by hand: a block with norms behind its sublayers, a pre-norm block whose norm it
    leaves ready, and one more of the first kind; the attention norms q over all heads, with biases and a
    gate, and the last block reads the first one's keys."""
    from types import SimpleNamespace

    from picolm_amd.engine.builder import parse_dtype
    from picolm_amd.engine.model import DecoderModel, LayerCall
    from picolm_amd.parts import LMHead, PreNormBlock, RMSNorm, SwiGLU, TokenEmbedding
    from picolm_amd.parts.base import Runtime
    from picolm_amd.parts.block import OutputNormBlock
    from picolm_amd.parts.recurrent import LinearAttention
    from picolm_amd.parts.sink_attention import SinkAttention
    from picolm_amd.weights import TensorDict
    from plain import belorax_plain as P
    D, V, H, G, d, dv, eps, mult = 40, 53, 4, 2, 10, 6, 1e-4, 0.8

    def attn(prefix, reads):
        return SinkAttention(prefix, D, H, G, d, dv, 0.4, eps, sink=False, proj_bias=True, norm_all=True, q_temp=(0.7, 9), reads_keys=reads)
    emb = TokenEmbedding("embed", V, D)
    blocks = [OutputNormBlock(attn("a.", False), RMSNorm("n0", D, eps), None, None, mult),
              PreNormBlock(RMSNorm("n1", D, eps), LinearAttention("r.", D, 2, 8, 6, eps, decay=[0.9, 0.6]), RMSNorm("n2", D, eps),
                           SwiGLU("f.", D, 24, names=("gate", "up", "down"))),
              OutputNormBlock(attn("b.", True), RMSNorm("n3", D, eps), SwiGLU("g.", D, 24, names=("gate", "up", "down")), RMSNorm("n4", D, eps), mult)]
    model = DecoderModel(SimpleNamespace(), emb, blocks, RMSNorm("final.norm", D, eps), LMHead("head", V, D, emb, tied=False),
                         [LayerCall(0), LayerCall(1), LayerCall(2, reads_cache_of=0)])
    gen = torch.Generator().manual_seed(1)
    w = {}
    for s in model.tensor_specs():
        one = len(s.shape) == 1 and not s.name.endswith(".b")
        w[s.name] = ((1.0 + 0.2 * torch.randn(*s.shape, generator=gen)) if one else torch.randn(*s.shape, generator=gen) /
                     (s.shape[-1] ** 0.5 if len(s.shape) == 2 and s.name != "embed" else 1.0)).to(torch.bfloat16)
    model.load(TensorDict(w), Runtime(torch.device("cuda:0"), parse_dtype(dtype)))
    W = bt.as_arrays(w)
    tokens = [int(t) for t in np.random.default_rng(4).integers(0, V, size=70)]

    def project(h, p, n, heads, norm):
        y = h @ W[p + n].T + W[p + n + ".b"]
        return P.heads_of(P.rms_norm(y, W[p + n + ".norm"], eps) if norm else y, heads)

    def attend(h, p, kv):
        q = project(h, p, "q", H, True) * P.query_temperature(len(h), dict(coef=0.7, every=9))[:, None, None]
        out = np.stack([P.causal_softmax(q[:, a] @ kv[0][:, a // 2].T * 0.4) @ kv[1][:, a // 2] for a in range(H)], axis=1).reshape(len(h), -1)
        return (out / (1 + np.exp(-(h @ W[p + "g"].T)))) @ W[p + "o"].T
    x = W["embed"][tokens]
    kv = project(x, "a.", "k", G, True), project(x, "a.", "v", G, False)
    x = x + mult * P.rms_norm(attend(x, "a.", kv), W["n0"], eps)
    h = P.rms_norm(x, W["n1"], eps)
    q, k, v = (P.heads_of(h @ W["r." + n].T, 2) for n in "qkv")
    o = P.rms_norm(P.decayed_state_walk(q, k, v, [0.9, 0.6]), W["r.norm"], eps).reshape(70, -1)
    x = x + (o * P.silu(h @ W["r.g"].T)) @ W["r.o"].T
    x = x + P.gated(P.rms_norm(x, W["n2"], eps), W, "f.")
    x = x + mult * P.rms_norm(attend(x, "b.", kv), W["n3"], eps)
    x = x + mult * P.rms_norm(P.gated(x, W, "g."), W["n4"], eps)
    want = P.rms_norm(x, W["final.norm"], eps) @ W["head"].T
    s = new_session(model, 256)
    assert bt.distance(run_whole(s, tokens), want) <= bt.LIMIT[dtype]
    [slot] = s.begin(1)
    got = [s.step([slot], [[t]]).double().cpu().numpy() for t in tokens]
    assert bt.distance(np.concatenate(got), want) <= bt.LIMIT[dtype]
    s.release([slot])


# ------------------------------------------------------------------------------ prompts, decoding, portions
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_prompt_decoding_and_portions(which, dtype):
    cfg, w, model = model_of(which, dtype)
    tokens = tokens_for(cfg, 150, 1)
    want = truth_of(which, 0, tokens)
    s = new_session(model, 1024)
    assert bt.near(run_whole(s, tokens), want, slice(None), dtype)
    # most of it at once, the rest one by one (past the page border at 128)
    [slot] = s.begin(1)
    got = s.step([slot], [tokens[:101]], [[0, 1, 2, 63, 64, 100]]).double().cpu().numpy()
    assert bt.near(got, want, [0, 1, 2, 63, 64, 100], dtype)
    for i in range(101, 150):
        got = s.step([slot], [[tokens[i]]]).double().cpu().numpy()
        assert bt.near(got, want, i, dtype), ("decoded", i)
    s.release([slot])
    # portions of several sizes, down to two tokens and one, every row wanted
    for sizes in ([2, 2, 3, 57, 1, 64, 21], [64, 64, 22], [1, 1, 2, 146], [149, 1], [36, 37, 38, 39]):
        assert sum(sizes) == 150
        [slot] = s.begin(1)
        at = 0
        for n in sizes:
            got = s.step([slot], [tokens[at:at + n]], [list(range(n))]).double().cpu().numpy()
            assert bt.near(got, want, slice(at, at + n), dtype), (sizes, "portion at", at)
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
    assert bt.distance(np.concatenate(parts), whole) <= (2e-5 if dtype == "float32" else 0.03)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "B"])
def test_a_long_prompt(which, dtype):
    """Several pages and several tiles of queries, prompts that the states are walked in chunks for, the
    last of them short; whole, in portions, and beside short requests in a batch, then decoded on."""
    cfg, w, model = model_of(which, dtype)
    tokens = tokens_for(cfg, 405, 8)
    want = truth_of(which, 0, tokens)
    s = new_session(model, 2048)
    assert bt.near(run_whole(s, tokens[:401]), want, slice(0, 401), dtype)
    [slot] = s.begin(1)
    rows = [0, 63, 64, 100]
    got = s.step([slot], [tokens[:101]], [rows]).double().cpu().numpy()
    assert bt.near(got, want, rows, dtype)
    got = s.step([slot], [tokens[101:401]], [list(range(300))]).double().cpu().numpy()
    assert bt.near(got, want, slice(101, 401), dtype)
    for i in range(401, 405):
        got = s.step([slot], [[tokens[i]]]).double().cpu().numpy()
        assert bt.near(got, want, i, dtype), ("decoded", i)
    s.release([slot])
    others = [tokens_for(cfg, n, 30 + n) for n in (10, 257)]
    slots = s.begin(3)
    got = s.step(slots, [tokens[:400]] + others).double().cpu().numpy()
    assert bt.near(got[0], want, 399, dtype)
    for i, q in enumerate(others):
        assert bt.near(got[1 + i], truth_of(which, 0, q), len(q) - 1, dtype), ("beside the long one", i)
    got = s.step(slots[:1], [[tokens[400]]]).double().cpu().numpy()
    assert bt.near(got, want, 400, dtype)
    s.release(slots)


# strong decays and weak ones, heads that turn in part, over a prompt long enough to be walked in chunks
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,vdim,dims", [(64, 96, 64), (128, 128, 32), (40, 24, 40), (200, 72, 10)])
def test_states_over_a_long_prompt_of_uneven_decays(dim, vdim, dims, dtype):
    cfg = one_layer(bt.retention(dim, vdim, [1.0, 0.0, 0.3, 0.999], bt.rotation(dims, 1000.0)), width=64)
    w = bt.make_weights(cfg, 4)
    tokens = tokens_for(cfg, 330, 9)
    want = bt.Truth(cfg, w, tokens)
    s = new_session(bt.load(cfg, w, dtype), 1024)
    assert bt.near(run_whole(s, tokens), want, slice(None), dtype)
    [slot] = s.begin(1)
    at = 0
    for n in (3, 259, 65, 1, 2):
        got = s.step([slot], [tokens[at:at + n]], [list(range(n))]).double().cpu().numpy()
        assert bt.near(got, want, slice(at, at + n), dtype), ("portion at", at)
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
        assert bt.near(got[at:at + n], truth[i], slice(0, n), dtype), ("prompt", i)
        at += n
    # and against each alone, much closer than the plain model is in bfloat16: what else is in the batch does not show
    alone = new_session(model, 512)
    at = 0
    for i, n in enumerate(lens):
        assert bt.distance(got[at:at + n], run_whole(alone, seqs[i][:n])) <= (2e-5 if dtype == "float32" else 0.03), ("alone", i)
        at += n
    # the shorter ones end earlier: after two steps the first two leave the batch
    live = list(range(len(seqs)))
    for j in range(n_dec):
        if j == 2:
            s.release([slots[0], slots[1]])
            live = live[2:]
        got = s.step([slots[i] for i in live], [[seqs[i][lens[i] + j]] for i in live]).double().cpu().numpy()
        for row, i in enumerate(live):
            assert bt.near(got[row], truth[i], lens[i] + j, dtype), ("step", j, "sequence", i)
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
        assert bt.near(got, want, rows, dtype), ("prompt", k)
        for i in range(cut, n):
            got = s.step([slot], [[tokens[i]]]).double().cpu().numpy()
            assert bt.near(got, want, i, dtype), ("sequence", k, "token", i)
        s.release([slot])
    # two sequences that swap slots between uses
    a, b = tokens_for(cfg, 40, 90), tokens_for(cfg, 66, 91)
    for order in ((a, b), (b, a)):
        slots = s.begin(2)
        got = s.step(slots, list(order)).double().cpu().numpy()
        for i, q in enumerate(order):
            assert bt.near(got[i], truth_of("A", 0, q), len(q) - 1, dtype)
        s.release(slots)


# ------------------------------------------------------------------------------ far keys, page borders, states
def ones_and_loud(w, name, by):
    """The norm behind the asking mixer with weight `by`: the branch outweighs the rows it is added to."""
    w[name] = torch.full_like(w[name], by - 1.0)


def lookup_attention(dim, asks, width=64):
    """Layers of attention of which layer `asks` looks a token's partner up while the others add nothing
    (their output products are zero); layers after the first read the first one's keys, past a
    retention that adds nothing either.  Token t + 700 has the first half of token t's embedding.  Keys
    read the first half of the width and queries are the keys' rows, so the score of two tokens with the
    same first half is as high as a token's with itself and far above the chance products of hundreds
    of other keys; what the partner contributes differs from the asking token's own contribution through
    the second half of the width (the values read it).  So the asking token's output rests on its
    partner wherever the partner stands."""
    half, heads, vdim = width // 2, 2, dim if dim == 64 else 16
    attn = lambda **kw: bt.layer(bt.attention(heads, 1, dim, vdim, 30.0 / dim, 0.1, 50, **kw))
    layers = [attn()] if asks == 0 else [attn(), bt.layer(bt.retention(6, 4, [0.9], bt.rotation(4)))] + [attn(kv_from=0) for _ in range(asks - 1)]
    cfg = bt.config(1400, width, layers, scale=1.0, mult=1.0)
    w = bt.make_weights(cfg, 5)
    w["embed"][700:, :half] = w["embed"][:700, :half]
    keys = torch.randn(dim, width, generator=torch.Generator().manual_seed(2), dtype=torch.float64) / half ** 0.5
    keys[:, half:] = 0
    for i, l in enumerate(layers):
        p = f"l{i}.mix."
        if i != asks:
            w[p + "o"] = torch.zeros_like(w[p + "o"])
        if l["type"] == "attention":
            w[p + "q"] = torch.cat([keys] * heads).to(torch.bfloat16)
            w[p + "q.norm"] = torch.ones_like(w[p + "q.norm"])
    w["l0.mix.k"], w["l0.mix.k.norm"] = keys.to(torch.bfloat16), torch.ones_like(w["l0.mix.k.norm"])
    w["l0.mix.v"][:, :half] = 0
    ones_and_loud(w, f"l{asks}.norm1", 16.0)
    return cfg, w


def lookup_latent(kv_rank, dim=48, vdim=16, heads=2, width=64):
    """The same over latents: all but the last eight entries of a latent read the first half of the
    width, the last eight (kept small, so that the others decide the latent's norm) the second half.
    The unrotated queries are W_uk of a head times the same rows that make the latent; values read the
    last eight entries; the rotated parts are small beside that."""
    keys, half = kv_rank - 8, width // 2
    rot_dim = 32 if kv_rank == 64 else 16      # keys of 96 over latents of 64 go through the matrix-core kernel in bfloat16
    cfg = bt.config(1400, width, [bt.layer(bt.latent(heads, dim, rot_dim, vdim, kv_rank, 30.0 / kv_rank, 10000.0, bt.yarn(4.0, 64, 8.0, 2.0)))],
                    scale=1.0, mult=1.0)
    w = bt.make_weights(cfg, 5)
    w["embed"][700:, :half] = w["embed"][:700, :half]
    p, dkv = "l0.mix.", w["l0.mix.dkv"]
    dkv[:keys, half:] = 0
    dkv[keys:kv_rank, :half] = 0
    dkv[keys:kv_rank] = (0.25 * dkv[keys:kv_rank].double()).to(torch.bfloat16)
    dkv[kv_rank:] = (0.2 * dkv[kv_rank:].double()).to(torch.bfloat16)
    w[p + "dkv.norm"] = torch.ones(kv_rank, dtype=torch.bfloat16)
    uk = torch.randn(heads * dim, kv_rank, generator=torch.Generator().manual_seed(2), dtype=torch.float64) / dim ** 0.5
    uk[:, keys:] = 0
    w[p + "uk"] = uk.to(torch.bfloat16)
    q = w[p + "q"].double().view(heads, dim + rot_dim, width)
    q[:, :dim] = (w[p + "uk"].double() @ (1.5 * dkv[:kv_rank].double())).view(heads, dim, width)
    q[:, dim:] *= 0.2
    w[p + "q"] = q.reshape(heads * (dim + rot_dim), width).to(torch.bfloat16)
    w[p + "uv"][:, :keys] = 0
    ones_and_loud(w, "l0.norm1", 16.0)
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


def asking_sequence(key, cfg, w, n, needle_at, seed):
    """n tokens whose last one's partner stands at `needle_at`, the plain model's logits of the last
    token, and a check that the test can tell: with the partner replaced by an unrelated token the
    logits differ by far more than rounding (tokens are drawn again until they do)."""
    if key in _FAR:
        return _FAR[key]
    while True:
        tokens = distinct_tokens(n, needle_at, cfg["vocab"], seed)
        want = bt.plain_logits(cfg, w, tokens)[-1]
        missed = bt.plain_logits(cfg, w, without_the_partner(tokens, needle_at, cfg["vocab"]))[-1]
        if bt.distance(missed, want) > 0.2:
            _FAR[key] = (tokens, want)
            return _FAR[key]
        seed += 1000


def ask_in_a_prompt_and_decoded(s, tokens, want, dtype, what):
    [slot] = s.begin(1)
    got = s.step([slot], [tokens]).double().cpu().numpy()
    assert bt.distance(got, want) <= bt.LIMIT[dtype], ("prompt",) + what
    s.release([slot])
    [slot] = s.begin(1)
    s.step([slot], [tokens[:-1]], [[]])
    got = s.step([slot], [tokens[-1:]]).double().cpu().numpy()
    assert bt.distance(got, want) <= bt.LIMIT[dtype], ("decoded",) + what
    s.release([slot])


PLACES = (0, 1, 63, 64, 65, 128, 383, 498)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,asks", [(20, 0), (64, 0), (20, 2), (64, 3)])
def test_one_far_key_among_hundreds(dim, asks, dtype):
    """The asking token is the last; the key it asks for lies hundreds back, at the first places of
    the sequence, and just before and after page borders; kept by the asking layer, or by the first
    one whose keys the asking layer reads.  Both in a prompt and decoded.  (Keys of 64 go through the
    matrix-core kernel in bfloat16, the others through the vector ALU.)"""
    cfg, w = lookup_attention(dim, asks)
    s = new_session(bt.load(cfg, w, dtype), 2048)
    for needle_at in PLACES:
        tokens, want = asking_sequence((dim, asks, needle_at), cfg, w, 500, needle_at, needle_at)
        ask_in_a_prompt_and_decoded(s, tokens, want, dtype, (needle_at,))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kv_rank", [40, 64])
def test_one_far_latent_among_hundreds(kv_rank, dtype):
    cfg, w = lookup_latent(kv_rank)
    s = new_session(bt.load(cfg, w, dtype), 2048)
    for needle_at in PLACES:
        tokens, want = asking_sequence(("latent", kv_rank, needle_at), cfg, w, 500, needle_at, needle_at)
        ask_in_a_prompt_and_decoded(s, tokens, want, dtype, (needle_at,))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,asks", [(20, 0), (64, 2)])
def test_a_key_that_was_decoded_and_is_asked_for_in_a_batch(dim, asks, dtype):
    """A short prompt, then single tokens until the asking one, in a batch with a longer sequence: the
    partner is a token of the prompt or a decoded one on either side of a page border."""
    cfg, w = lookup_attention(dim, asks)
    s = new_session(bt.load(cfg, w, dtype), 1024)
    beside = distinct_tokens(300, 3, cfg["vocab"], 77)
    n = 150
    for needle_at in (2, 20, 63, 64, 127, 128):
        tokens, want = asking_sequence(("decoded", dim, asks, needle_at), cfg, w, n, needle_at, needle_at)
        slots = s.begin(2)
        s.step(slots, [tokens[:8], beside[:300 - (n - 8)]], [[], []])
        for i in range(8, n):
            got = s.step(slots, [[tokens[i]], [beside[300 - n + i]]]).double().cpu().numpy()
        assert bt.distance(got[0], want) <= bt.LIMIT[dtype], needle_at
        s.release(slots)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dims", [2, 16])
def test_a_far_token_in_a_state_that_keeps(dims, dtype):
    """A state that keeps everything: what a token wrote hundreds of tokens ago, in the first chunk of a
    prompt, at a chunk's edge, or in an earlier step, is in the output of the last."""
    dim, n = 96, 300
    cfg = one_layer(bt.retention(dim, 24, [1.0], bt.rotation(dims, 1e6)), width=64, scale=1.0, mult=1.0)
    w = bt.make_weights(cfg, 6)
    p = "l0.mix."
    # entries 8 to 15 of a rare token, 60, make a strong key and value; entries 0 to 7 of the asking token, 59, the query that meets it
    key = 4.0 * w[p + "k"][:, :8].double()
    w[p + "q"] = w[p + "k"].clone()
    w[p + "k"][:, :8], w[p + "k"][:, 8:16] = 0, key.to(torch.bfloat16)
    w[p + "q"][:, :8], w[p + "q"][:, 8:16] = key.to(torch.bfloat16), 0
    w[p + "v"][:, 8:16] = (4.0 * w[p + "v"][:, 8:16].double()).to(torch.bfloat16)
    w["embed"][:60, :16] = (0.1 * w["embed"][:60, :16].double()).to(torch.bfloat16)
    w["embed"][60], w["embed"][60, 8:16], w["embed"][59, :8] = 0, 3.0, 3.0
    ones_and_loud(w, "l0.norm1", 8.0)
    s = new_session(bt.load(cfg, w, dtype), 1024)
    rng = np.random.default_rng(1)
    for at in (0, 1, 63, 64, 65, 255, 256, 298):
        tokens = [int(t) for t in rng.integers(0, 59, size=n)]
        tokens[-1] = 59
        without = list(tokens)
        tokens[at] = 60
        want = bt.plain_logits(cfg, w, tokens)[-1]
        assert bt.distance(bt.plain_logits(cfg, w, without)[-1], want) > 0.2, "the token must count"
        ask_in_a_prompt_and_decoded(s, tokens, want, dtype, (at,))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dims", [8, 30])
def test_a_state_tells_positions_apart_by_the_rotation(dims, dtype):
    """With decays of one, where a token stands shows through the rotation alone: two sequences that
    differ in the order of their tokens, their last token's logits apart in the plain model and each met."""
    cfg = one_layer(bt.retention(30, 12, [1.0, 1.0], bt.rotation(dims, 50.0)), width=64)
    w = bt.make_weights(cfg, 8)
    ones_and_loud(w, "l0.norm1", 16.0)
    a = tokens_for(cfg, 130, 3)
    b = a[64:128] + a[:64] + a[128:]
    want = [bt.Truth(cfg, w, t) for t in (a, b)]
    assert bt.distance(want[0][-1], want[1][-1]) > 0.2
    s = new_session(bt.load(cfg, w, dtype), 512)
    for t, truth in zip((a, b), want):
        assert bt.near(run_whole(s, t)[-1], truth, len(t) - 1, dtype)
        [slot] = s.begin(1)
        s.step([slot], [t[:100]], [[]])
        for i in range(100, 130):
            got = s.step([slot], [[t[i]]]).double().cpu().numpy()
        assert bt.near(got, truth, 129, dtype)
        s.release([slot])


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_tokens_of_a_sequence(dtype):
    """Sequences of one, two and three tokens, alone and in one batch."""
    cfg, w, model = model_of("C", dtype)
    s = new_session(model, 512)
    seqs = [tokens_for(cfg, n, 60 + n) for n in (1, 2, 3, 1)]
    for q in seqs:
        assert bt.near(run_whole(s, q), truth_of("C", 0, q), slice(None), dtype)
    slots = s.begin(len(seqs))
    got = s.step(slots, seqs).double().cpu().numpy()
    for i, q in enumerate(seqs):
        assert bt.near(got[i], truth_of("C", 0, q), len(q) - 1, dtype)
    s.release(slots)


# ------------------------------------------------------------------------------ long decoding
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "B"])
def test_long_decoding_through_recorded_steps(which, dtype):
    """Three sequences decoded 200 tokens, over page borders; from the second step of
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
            assert bt.near(got[i], truth[i], n + j, dtype), ("step", j, "sequence", i)
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
    return bt.write_folder(str(tmp_path_factory.mktemp("belorax") / "a"), bt.CONFIGS["A"], bt.make_weights(bt.CONFIGS["A"], 0))


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_entry_point(dtype, folder_a):
    import picolm_amd
    prompts = [tokens_for(bt.CONFIGS["A"], n, 50 + n) for n in (4, 9, 66)]
    got = picolm_amd.generate(folder_a, prompts, max_new_tokens=10, stop_ids=(), dtype=dtype)
    for p, r in zip(prompts, got):
        assert len(r.tokens) == 10 and r.finish == "length"
        seq = list(p)
        for k in range(10):
            lg = truth_of("A", 0, seq)[-1]
            top2 = np.sort(lg)[-2:]
            if top2[1] - top2[0] < 4 * bt.LIMIT[dtype] * lg.std():
                break                              # a near tie: either choice is right
            assert r.tokens[k] == int(np.argmax(lg)), (k, r.tokens)
            seq.append(r.tokens[k])


def test_trace_replay_and_command_line(folder_a, tmp_path):
    """bin/trace_run on a folder: a prompt, single tokens and a second request that joins later in a
    slot that was given back; bin/picolm generates from the same folder."""
    cfg = bt.CONFIGS["A"]
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
    assert bt.near(read(0), ta, [0, 16], "float32")
    assert bt.near(read(1), ta, 17, "float32")
    assert not os.path.exists(os.path.join(out, "2.f32"))
    assert bt.near(read(3), ta, 19, "float32")
    assert bt.near(read(4), tb, 8, "float32")
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "picolm"), folder_a, "-p", " ".join(map(str, b)), "-n", "4", "-t", "0",
                        "--dtype", "float32"], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert len(r.stdout.split()) == 4
    assert int(r.stdout.split()[0]) == int(np.argmax(tb[-1]))
