"""Belorax without a GPU: the configuration's faults by key, the cache entries that its layers ask
for, the parts' own checks, and closed forms that pin the plain model of tests/plain/belorax_plain.py
itself."""
import copy
import json
import math

import numpy as np
import pytest
import torch

import belorax_tiny as bt
from picolm_amd.config import ConfigError, resolve
from picolm_amd.config.belorax import BeloraxConfig, RotationConfig
from picolm_amd.engine.builder import build_from_config_dict
from plain import belorax_plain as P


def test_the_registry_knows_the_name_and_the_configuration_round_trips():
    for cfg in bt.CONFIGS.values():
        assert resolve(cfg).name == "Belorax"
        typed = BeloraxConfig.from_dict(cfg)
        assert BeloraxConfig.from_dict(typed.to_dict()) == typed
        assert BeloraxConfig.from_dict(json.loads(json.dumps(typed.to_dict()))) == typed
        assert typed.vocab_size == cfg["vocab"] and typed.hidden_size == cfg["width"]


def mixer_path(i, *keys):
    return ("layers", i, "mixer") + keys


@pytest.mark.parametrize("path,value,names", [
    (("vocab",), None, "vocab"), (("width",), 0, "width"), (("norm", "eps"), 0.0, "norm.eps"), (("layers",), [], "layers"),
    (("embedding",), 3.0, "embedding"), (("embedding", "scale"), "x", "embedding.scale"), (("residual_mult",), "x", "residual_mult"),
    (("residual_mult",), 0, "residual_mult"), (("layers", 0, "type"), "retention2", "layers[0].type"), (("layers", 3, "mixer"), None, "layers[3].mixer"),
    (mixer_path(0, "decay"), [0.5], "layers[0].mixer.decay"), (mixer_path(0, "decay"), None, "layers[0].mixer.decay"),
    (mixer_path(0, "decay"), [0.5, 0.5, 1.5], "layers[0].mixer.decay"), (mixer_path(0, "vdim"), 0, "layers[0].mixer.vdim"),
    (mixer_path(0, "dim"), 300, "layers[0].mixer.dim"), (mixer_path(0, "rot", "dims"), 7, "layers[0].mixer.rot.dims"),
    (mixer_path(0, "rot", "dims"), 16, "layers[0].mixer.rot.dims"), (mixer_path(0, "rot", "base"), 0.0, "layers[0].mixer.rot.base"),
    (mixer_path(1, "heads"), None, "layers[1].mixer.heads"), (mixer_path(1, "kv_heads"), 4, "layers[1].mixer.kv_heads"),
    (mixer_path(1, "scale"), 0.0, "layers[1].mixer.scale"), (mixer_path(1, "dim"), 2000, "layers[1].mixer.dim"),
    (mixer_path(1, "q_temp", "every"), 0, "layers[1].mixer.q_temp.every"), (mixer_path(1, "q_temp", "coef"), None, "layers[1].mixer.q_temp.coef"),
    (mixer_path(2, "kv_from"), 2, "layers[2].mixer.kv_from"), (mixer_path(4, "kv_from"), 2, "layers[4].mixer.kv_from"),
    (mixer_path(4, "kv_from"), 3, "layers[4].mixer.kv_from"), (mixer_path(4, "vdim"), 13, "layers[4].mixer.kv_from"),
    (mixer_path(4, "kv_heads"), 3, "layers[4].mixer.kv_from"), (mixer_path(4, "dim"), 10, "layers[4].mixer.kv_from"),
    (mixer_path(3, "kv_rank"), 0, "layers[3].mixer.kv_rank"), (mixer_path(3, "rot", "dims"), 6, "layers[3].mixer.rot.dims"),
    (mixer_path(3, "rot"), None, "layers[3].mixer.rot"), (mixer_path(3, "kv_rank"), 2000, "layers[3].mixer.kv_rank"),
    (mixer_path(3, "rot", "scaling", "factor"), None, "layers[3].mixer.rot.scaling.factor"),
    (mixer_path(3, "rot", "scaling", "slow"), 0.0, "layers[3].mixer.rot.scaling.slow"), (mixer_path(3, "rot", "base"), 1.0, "layers[3].mixer.rot.base"),
    (("layers", 0, "mlp", "kind"), "mixed", "layers[0].mlp.kind"), (("layers", 0, "mlp", "ff"), None, "layers[0].mlp.ff"),
    (("layers", 1, "mlp", "router", "top"), 7, "layers[1].mlp.router.top"), (("layers", 1, "mlp", "expert"), None, "layers[1].mlp.expert"),
])
def test_a_fault_names_its_key(path, value, names):
    cfg = copy.deepcopy(bt.CONFIG_A)
    at = cfg
    for key in path[:-1]:
        at = at[key]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    with pytest.raises(ConfigError) as e:
        BeloraxConfig.from_dict(cfg)
    assert names in str(e.value)


def test_a_layer_may_leave_out_what_has_a_usual_value():
    cfg = copy.deepcopy(bt.CONFIG_A)
    del cfg["layers"][0]["mixer"]["rot"]
    for l in cfg["layers"]:
        if l["type"] == "attention":
            del l["mixer"]["q_temp"]
    cfg["layers"][3]["mixer"]["rot"]["scaling"] = None
    typed = BeloraxConfig.from_dict(cfg)
    assert typed.layers[0].mixer.rot is None and typed.layers[1].mixer.q_temp is None and typed.layers[3].mixer.rot.scaling is None
    assert BeloraxConfig.from_dict(typed.to_dict()) == typed


def test_what_the_layers_ask_of_the_cache_and_the_checkpoint():
    model = build_from_config_dict(bt.CONFIG_A)
    assert [c.reads_cache_of for c in model.order] == [None, None, 1, None, 1, None]
    assert [(b.kv, b.state is not None, b.writes) for b in model.bindings] == [
        (None, True, True), ((0, 0), False, True), ((0, 0), False, False), ((1, 0), False, True), ((0, 0), False, False), (None, True, True)]
    kv = [(g.n_entries, g.n_kv_heads, g.head_dim, g.value_dim, g.window) for g in model.cache_spec.kv_groups]
    assert kv == [(1, 2, 20, 12, 0), (1, 1, 28, 20, 0)]
    assert [g.shape for g in model.cache_spec.state_groups] == [(3 * 14 * 20,), (2 * 18 * 10,)]
    assert all(g.dtype == torch.float32 for g in model.cache_spec.state_groups)
    for cfg in bt.CONFIGS.values():
        specs = {s.name: tuple(s.shape) for s in build_from_config_dict(cfg).tensor_specs() if not s.optional or s.name == "head"}
        assert specs == bt.tensor_shapes(cfg)


def test_layers_that_turn_alike_share_their_tables():
    cfg = bt.config(50, 16, [bt.layer(bt.retention(8, 4, [0.5], bt.rotation(4))), bt.layer(bt.retention(6, 4, [0.5], bt.rotation(4))),
                             bt.layer(bt.latent(2, 4, 4, 4, 6, 0.5))])
    a, b, c = (blk.mixer.position for blk in build_from_config_dict(cfg).blocks)
    assert a is b and a.style == "half" and c.style == "pairwise" and c is not a


def test_the_parts_refuse_what_does_not_go_together():
    from picolm_amd.parts.block import OutputNormBlock
    from picolm_amd.parts.norm import RMSNorm
    from picolm_amd.parts.position import RotaryEmbedding
    from picolm_amd.parts.recurrent import LinearAttention
    from picolm_amd.parts.sink_attention import SinkAttention
    with pytest.raises(ValueError):
        LinearAttention("m.", 16, 2, 8, 8, 1e-5, decay=[0.5, 0.5], position=RotaryEmbedding(10, 100.0))
    with pytest.raises(ValueError):
        LinearAttention("m.", 16, 2, 8, 8, 1e-5, decay=[0.5, 0.5], silu_qkv=True, position=RotaryEmbedding(8, 100.0))
    with pytest.raises(ValueError):
        SinkAttention("m.", 16, 2, 1, 8, 8, 0.3, 1e-5, q_temp=(0.5, 0.0))
    mixer = SinkAttention("m.", 16, 2, 1, 8, 8, 0.3, 1e-5)
    with pytest.raises(ValueError):
        OutputNormBlock(mixer, RMSNorm("n", 16, 1e-5), None, RMSNorm("n2", 16, 1e-5))
    with pytest.raises(ValueError):
        OutputNormBlock(mixer, RMSNorm("n", 16, 1e-5), None, None, 0.0)


def test_a_layer_that_reads_keys_has_no_tensors_of_them():
    from picolm_amd.parts.sink_attention import SinkAttention
    m = SinkAttention("m.", 16, 4, 2, 6, 5, 0.3, 1e-5, sink=False, gate=True, proj_bias=True, reads_keys=True)
    names = {s.name: tuple(s.shape) for s in m.all_specs()}
    assert names == {"m.q": (24, 16), "m.g": (20, 16), "m.o": (16, 20), "m.q.norm": (6,), "m.q.b": (24,)}


# ------------------------------------------------------------------------------ closed forms of the plain model
def test_the_plain_norms():
    x = np.array([[1.0, 2.0, 3.0, 6.0]])
    w = np.array([1.0, 2.0, 0.5, 0.0])
    assert np.allclose(P.rms_norm(x, w, 0.5), x / math.sqrt(12.5 + 0.5) * w)
    assert np.allclose(P.rms_norm_about_one(x, w, 0.5), x / math.sqrt(12.5 + 0.5) * (1 + w))
    assert np.allclose(P.unit_rms(x, 3.5), x / 4.0)


def test_the_plain_rotation_pairs_halves_or_neighbours():
    rot = dict(base=100.0, dims=4)                                    # frequencies 1 and 0.1
    x = np.zeros((4, 1, 5))
    x[3, 0] = [1.0, 2.0, 3.0, 4.0, 9.0]                               # the fifth entry is not turned
    c, s, c2, s2 = math.cos(3.0), math.sin(3.0), math.cos(0.3), math.sin(0.3)
    assert np.allclose(P.rotate(x, rot, True)[3, 0], [c - 3 * s, 2 * c2 - 4 * s2, 3 * c + s, 4 * c2 + 2 * s2, 9.0])
    assert np.allclose(P.rotate(x, rot, False)[3, 0], [c - 2 * s, 2 * c + s, 3 * c2 - 4 * s2, 4 * c2 + 3 * s2, 9.0])
    first = np.array([[[1.0, 2.0, 3.0, 4.0]]])
    assert np.allclose(P.rotate(first, rot, True), first)
    # base 4, eight entries: frequencies 1, 2^-1/2, 1/2, 2^-3/2; a pair turns t times in 2 pi 2^n t positions at i = 2 n: with an
    # `original` of 8 pi sqrt(2), `fast` 4 ends at (log2(4 sqrt(2)) - 2) 2 = 1 and `slow` 1 at 5, so the ramp runs from pair 1 to pair 5
    rot = dict(base=4.0, dims=8, scaling=bt.yarn(5.0, 8 * math.pi * 2 ** 0.5, 4.0, 1.0))
    f, mag = P.rotary_frequencies(rot)
    plain = 4.0 ** (-np.arange(4) / 4.0)
    ramp = np.array([0.0, 0.0, 0.25, 0.5])
    assert np.allclose(f, plain / 5 * ramp + plain * (1 - ramp), rtol=1e-9) and math.isclose(mag, 0.1 * math.log(5.0) + 1.0)


def test_the_product_side_frequencies_are_the_plain_ones():
    from picolm_amd.parts.position import rotary_inv_freq, rotary_magnitude
    for rot in (dict(base=4.0, dims=8, scaling=bt.yarn(5.0, 15.0, 2.0, 0.5)), dict(base=30000.0, dims=28, scaling=bt.yarn(3.0, 300, 32.0, 1.0)),
                dict(base=77.0, dims=6), dict(base=500.0, dims=32, scaling=bt.yarn(2.0, 100, 1.0, 1.0))):
        c = RotationConfig.from_dict(rot, "")
        f, mag = P.rotary_frequencies(rot)
        assert np.allclose(rotary_inv_freq(c.dims, c.base, c.scaling).numpy(), f, rtol=1e-12)
        assert math.isclose(rotary_magnitude(c.scaling), mag)


def test_the_plain_temperature_steps_where_a_stretch_ends():
    t = P.query_temperature(9, dict(coef=0.5, every=3))
    assert np.allclose(t, 1 + 0.5 * np.log([1, 1, 2, 2, 2, 3, 3, 3, 4]))
    assert np.allclose(P.query_temperature(5, dict(coef=-1.0, every=2.5)), 1 - np.log([1, 1, 2, 2, 3]))
    assert np.allclose(P.query_temperature(4, None), 1.0)


def test_the_plain_softmax_sees_no_later_key():
    p = P.causal_softmax(np.log(np.array([[2.0, 9.0, 9.0], [1.0, 3.0, 9.0], [1.0, 2.0, 5.0]])))
    assert np.allclose(p, [[1, 0, 0], [0.25, 0.75, 0], [0.125, 0.25, 0.625]])


def test_the_plain_state_decays_before_it_takes_the_token_and_is_read_after():
    q, k, v = np.array([[[1.0, 2.0]], [[3.0, 1.0]]]), np.array([[[1.0, 0.0]], [[2.0, 5.0]]]), np.array([[[7.0]], [[11.0]]])
    out = P.decayed_state_walk(q, k, v, [0.5])                         # (the first token's decay meets a state of zeros)
    assert np.allclose(out[:, 0, 0], [7.0, 3.0 * (0.5 * 7 + 2 * 11) + 1.0 * (5 * 11)])


def one_layer(mixer, mlp=None, width=16, **kw):
    return bt.config(50, width, [bt.layer(mixer, mlp)], **kw)


def test_the_plain_retention_of_two_tokens():
    rng = np.random.default_rng(0)
    h = rng.normal(size=(2, 16))
    mixer = bt.retention(4, 6, [0.5, 0.25], bt.rotation(2, 7.0))        # entry 0 turns with entry 1, by one radian a position
    W = bt.as_arrays(bt.make_weights(one_layer(mixer), 3))
    p = "l0.mix."
    q, k, v = ((h @ W[p + n].T).reshape(2, 2, -1) for n in "qkv")
    R = np.eye(4)
    R[:2, :2] = [[math.cos(1), -math.sin(1)], [math.sin(1), math.cos(1)]]
    y = []
    for a, d in enumerate((0.5, 0.25)):
        o = d * ((R @ q[1, a]) @ k[0, a] / 2) * v[0, a] + (q[1, a] @ k[1, a] / 2) * v[1, a]
        y.append(o / np.sqrt((o ** 2).mean() + 0.3))
    g = h[1] @ W[p + "g"].T
    got = P.retention(h, W, p, mixer[1], 0.3)
    assert np.allclose(got[1], W[p + "o"] @ (np.concatenate(y) * g / (1 + np.exp(-g))))


def test_the_plain_attention_of_one_token_gives_its_value():
    h = np.random.default_rng(2).normal(size=(1, 16))
    mixer = bt.attention(4, 2, 6, 5, 0.5)
    W = bt.as_arrays(bt.make_weights(one_layer(mixer), 7))
    p = "l0.mix."
    v = (h[0] @ W[p + "v"].T).reshape(2, 5)
    kv = P.attention_keys(h, W, p, mixer[1], 1e-5)
    assert np.allclose(P.attention(h, W, p, mixer[1], 1e-5, kv)[0], W[p + "o"] @ np.concatenate([v[0], v[0], v[1], v[1]]))
    assert np.allclose((kv[0][0] / W[p + "k.norm"] * np.sqrt(((h[0] @ W[p + "k"].T).reshape(2, 6) ** 2).mean(1) + 1e-5)[:, None]).reshape(-1),
                       h[0] @ W[p + "k"].T)


def test_the_plain_attention_weighs_by_temperature_and_scale():
    h = np.random.default_rng(3).normal(size=(2, 16))
    kind, m = bt.attention(2, 1, 6, 5, 0.5, 0.8, 2)
    W = bt.as_arrays(bt.make_weights(one_layer((kind, m)), 9))
    p = "l0.mix."
    k, v = P.attention_keys(h, W, p, m, 1e-5)
    out = []
    for a in range(2):
        q = h[1] @ W[p + "q"][6 * a:6 * a + 6].T
        q = q / np.sqrt((q ** 2).mean() + 1e-5) * W[p + "q.norm"] * (1 + 0.8 * math.log(2))
        e = np.exp([0.5 * q @ k[0, 0], 0.5 * q @ k[1, 0]])
        out.append((e[0] * v[0, 0] + e[1] * v[1, 0]) / e.sum())
    assert np.allclose(P.attention(h, W, p, m, 1e-5, (k, v))[1], W[p + "o"] @ np.concatenate(out))


def test_the_plain_latent_attention_of_two_tokens():
    h = np.random.default_rng(4).normal(size=(2, 16))
    kind, m = bt.latent(2, 3, 4, 5, 6, 0.7, 9.0, bt.yarn(2.0, 30, 2.0, 0.5))
    W = bt.as_arrays(bt.make_weights(one_layer((kind, m)), 11))
    p = "l0.mix."
    f, mag = P.rotary_frequencies(m["rot"])
    R = np.zeros((4, 4))
    for i in range(2):
        R[2 * i:2 * i + 2, 2 * i:2 * i + 2] = [[math.cos(f[i]), -math.sin(f[i])], [math.sin(f[i]), math.cos(f[i])]]
    low = h @ W[p + "dkv"].T
    c = low[:, :6] / np.sqrt((low[:, :6] ** 2).mean(1, keepdims=True) + 1e-5) * W[p + "dkv.norm"]
    out = []
    for a in range(2):
        q = h[1] @ W[p + "q"][7 * a:7 * a + 7].T
        uk, uv = W[p + "uk"][3 * a:3 * a + 3], W[p + "uv"][5 * a:5 * a + 5]
        # the token's own rotation and its key's cancel; against the first token the query is one position on
        s = [q[:3] @ uk @ c[0] + mag * mag * (R @ q[3:]) @ low[0, 6:], q[:3] @ uk @ c[1] + mag * mag * q[3:] @ low[1, 6:]]
        e = np.exp(0.7 * np.array(s))
        out.append(uv @ (e[0] * c[0] + e[1] * c[1]) / e.sum())
    assert np.allclose(P.latent_attention(h, W, p, m, 1e-5)[1], W[p + "o"] @ np.concatenate(out))


def test_the_plain_experts_are_weighed_by_their_scores_as_they_are():
    h = np.random.default_rng(5).normal(size=(1, 16))
    mlp = bt.moe(4, 2, 3)
    W = bt.as_arrays(bt.make_weights(one_layer(bt.attention(1, 1, 4, 4, 0.5), mlp), 13))
    p = "l0.mlp."
    z = h[0] @ W[p + "router"].T
    s = np.exp(z) / np.exp(z).sum()
    best = np.argsort(-s)[:2]
    want = sum(s[e] * P.gated(h, W, f"{p}e{e}.")[0] for e in best)
    assert s[best].sum() < 0.98 and np.allclose(P.routed_experts(h, W, p, mlp)[0], want)
    assert math.isclose(P.router_margins(h, W, p, mlp)[0], z[best[1]] - np.sort(z)[1])


def test_the_plain_layer_adds_the_normed_branch_times_the_factor():
    cfg = one_layer(bt.attention(2, 1, 6, 5, 0.5), bt.dense(7), scale=3.0, mult=0.4, eps=0.1)
    W = bt.as_arrays(bt.make_weights(cfg, 15))
    x = 3.0 * W["embed"][[9]]
    y = np.tile((x @ W["l0.mix.v"].T), 2) @ W["l0.mix.o"].T            # one token: its value, for both heads
    x = x + 0.4 * y / np.sqrt((y ** 2).mean() + 0.1) * (1 + W["l0.norm1"])
    g = x @ W["l0.mlp.gate"].T
    y = (g / (1 + np.exp(-g)) * (x @ W["l0.mlp.up"].T)) @ W["l0.mlp.down"].T
    x = x + 0.4 * y / np.sqrt((y ** 2).mean() + 0.1) * (1 + W["l0.norm2"])
    want = (x / np.sqrt((x ** 2).mean() + 0.1) * (1 + W["final.norm"])) @ W["head"].T
    logits, after = P.forward(cfg, W, [9], return_layers=True)
    assert np.allclose(logits, want) and np.allclose(after[0], x)


def test_every_tensor_and_constant_shows_in_the_plain_logits():
    cfg = bt.CONFIG_A
    w = bt.make_weights(cfg, 0)
    tokens = [int(t) for t in np.random.default_rng(0).integers(0, cfg["vocab"], size=60)]
    base = bt.plain_logits(cfg, w, tokens)
    for name, t in w.items():
        changed = dict(w)
        changed[name] = (t.double() * 1.3 + 0.1 * torch.arange(t.numel(), dtype=torch.float64).reshape(t.shape).remainder(7)).to(torch.bfloat16)
        # (the logits' common part is taken off: a change of the head that every row shares would not show)
        assert bt.distance(bt.plain_logits(cfg, changed, tokens), base) > 1e-4, name
    for path, value in [(("embedding", "scale"), 3.0), (("norm", "eps"), 0.3), (("residual_mult",), 0.6), (mixer_path(0, "decay", 1), 0.9),
                        (mixer_path(0, "rot", "base"), 100.0), (mixer_path(0, "rot", "dims"), 6), (mixer_path(1, "scale"), 0.5),
                        (mixer_path(1, "q_temp", "coef"), 0.5), (mixer_path(1, "q_temp", "every"), 14), (mixer_path(2, "q_temp", "every"), 28),
                        (mixer_path(4, "scale"), 0.4), (mixer_path(3, "scale"), 0.4), (mixer_path(3, "rot", "base"), 300.0),
                        (mixer_path(3, "rot", "scaling", "factor"), 9.0), (mixer_path(3, "rot", "scaling", "original"), 20),
                        (mixer_path(3, "rot", "scaling", "fast"), 4.0), (mixer_path(3, "rot", "scaling", "slow"), 0.05),
                        (("layers", 1, "mlp", "router", "top"), 3)]:
        other = copy.deepcopy(cfg)
        at = other
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        assert bt.distance(bt.plain_logits(other, w, tokens), base) > 1e-4, path
    # what only the eps inside a norm lets show: scores that are not divided by their sum, keys times dim^(-1/2)
    kept, P.router_scores = P.router_scores, lambda h, W, p: 2.0 * kept(h, W, p)
    try:
        assert bt.distance(bt.plain_logits(cfg, w, tokens), base) > 1e-3
    finally:
        P.router_scores = kept
    walk, P.decayed_state_walk = P.decayed_state_walk, lambda q, k, v, decay: walk(q, 2.0 * k, v, decay)
    try:
        assert bt.distance(bt.plain_logits(cfg, w, tokens), base) > 1e-3
    finally:
        P.decayed_state_walk = walk
