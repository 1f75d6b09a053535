"""Zalalix without a GPU: the configuration's faults by key, the cache entries that its layers ask
for, the planning of decode steps over a window and kept first tokens, and closed forms that pin the
plain model of tests/plain/zalalix_plain.py itself."""
import copy
import json
import math

import numpy as np
import pytest
import torch

import zalalix_tiny as zt
from host_engine import G, host_engine
from picolm_amd.config import ConfigError, resolve
from picolm_amd.config.zalalix import ZalalixConfig
from picolm_amd.engine.builder import build_from_config_dict
from plain import zalalix_plain as P
from plan_reference import decode_pages_per_chunk


def test_the_registry_knows_the_name_and_the_configuration_round_trips():
    for cfg in zt.CONFIGS.values():
        assert resolve(cfg).name == "Zalalix"
        typed = ZalalixConfig.from_dict(cfg)
        assert ZalalixConfig.from_dict(typed.to_dict()) == typed
        assert ZalalixConfig.from_dict(json.loads(json.dumps(typed.to_dict()))) == typed
        assert typed.vocab_size == cfg["vocab"] and typed.hidden_size == cfg["width"]


LEFT, RIGHT = ("layers", 0, "mixer", "left"), ("layers", 0, "mixer", "right")


@pytest.mark.parametrize("path,value,names", [
    (("vocab",), None, "vocab"), (("width",), 0, "width"), (("norm", "eps"), 0.0, "norm.eps"), (("layers",), [], "layers"),
    (("embedding",), 3.0, "embedding"), (("embedding", "scale"), "x", "embedding.scale"),
    (("layers", 0, "type"), "lightning2", "layers[0].type"), (("layers", 0, "mixer", "left"), None, "layers[0].mixer.left"),
    (LEFT + ("heads",), None, "layers[0].mixer.left.heads"), (LEFT + ("kv_heads",), 4, "layers[0].mixer.left.kv_heads"),
    (LEFT + ("scale",), 0.0, "layers[0].mixer.left.scale"), (LEFT + ("softcap",), -1.0, "layers[0].mixer.left.softcap"),
    (LEFT + ("mask", "size"), 0, "layers[0].mixer.left.mask.size"), (LEFT + ("mask", "keep_first"), -1, "layers[0].mixer.left.mask.keep_first"),
    (LEFT + ("rot", "dims"), 7, "layers[0].mixer.left.rot.dims"), (LEFT + ("rot", "dims"), 22, "layers[0].mixer.left.rot.dims"),
    (LEFT + ("rot", "base"), 0.0, "layers[0].mixer.left.rot.base"), (LEFT + ("dim",), 2000, "layers[0].mixer.left.dim"),
    (LEFT + ("rot", "scaling", "factor"), None, "layers[0].mixer.left.rot.scaling.factor"),
    (LEFT + ("rot", "scaling", "high"), 0.5, "layers[0].mixer.left.rot.scaling.high"),
    (RIGHT + ("tau",), 0.0, "layers[0].mixer.right.tau"), (RIGHT + ("tau",), None, "layers[0].mixer.right.tau"),
    (RIGHT + ("dim",), 300, "layers[0].mixer.right.dim"), (("layers", 0, "mixer", "left_scale"), "x", "layers[0].mixer.left_scale"),
    (("layers", 1, "mixer", "decay"), [0.5], "layers[1].mixer.decay"), (("layers", 1, "mixer", "decay"), None, "layers[1].mixer.decay"),
    (("layers", 1, "mixer", "decay"), [0.5, 1.5], "layers[1].mixer.decay"), (("layers", 2, "mixer", "vdim"), 0, "layers[2].mixer.vdim"),
    (("layers", 0, "mlp", "kind"), "moe", "layers[0].mlp.kind"), (("layers", 0, "mlp", "ff"), None, "layers[0].mlp.ff"),
])
def test_a_fault_names_its_key(path, value, names):
    cfg = copy.deepcopy(zt.CONFIG_A)
    at = cfg
    for key in path[:-1]:
        at = at[key]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    with pytest.raises(ConfigError) as e:
        ZalalixConfig.from_dict(cfg)
    assert names in str(e.value)


def test_a_layer_may_leave_out_what_has_a_usual_value():
    cfg = copy.deepcopy(zt.CONFIG_A)
    left = cfg["layers"][0]["mixer"]["left"]
    for key in ("kv_heads", "scale", "softcap", "mask", "rot"):
        del left[key]
    typed = ZalalixConfig.from_dict(cfg)
    l = typed.layers[0].mixer.left
    assert (l.kv_heads, l.scale, l.softcap, l.window, l.keep_first, l.rot) == (6, 20 ** -0.5, 0.0, 0, 0, None)
    assert ZalalixConfig.from_dict(typed.to_dict()) == typed


def test_what_the_layers_ask_of_the_cache_and_the_checkpoint():
    model = build_from_config_dict(zt.CONFIG_A)
    assert [c.block for c in model.order] == [0, 1, 2, 3]
    assert [(b.kv is not None, b.state is not None) for b in model.bindings] == [(True, True), (False, True), (False, True), (True, True)]
    kv = {(g.n_kv_heads, g.head_dim, g.value_dim, g.window, g.keep_first): g.keeps_all for g in model.cache_spec.kv_groups}
    assert kv == {(2, 20, 12, 37, 5): True, (3, 14, 18, 70, 3): True}
    assert [g.shape for g in model.cache_spec.state_groups] == [(3 * 10 * 14,), (2 * 12 * 20,), (3 * 18 * 10,), (2 * 24 * 8,)]
    assert all(g.dtype == torch.float32 for g in model.cache_spec.state_groups)
    for cfg in zt.CONFIGS.values():
        shapes = zt.tensor_shapes(cfg)
        built = build_from_config_dict(cfg)
        specs = {s.name: tuple(s.shape) for s in built.tensor_specs() if s.name != "head"}
        assert specs == {k: v for k, v in shapes.items() if k != "head"}
        # without `rank` in the configuration the checkpoint's tensors say it
        bare = copy.deepcopy(cfg)
        for l in bare["layers"]:
            if l["type"] == "parallel":
                del l["mixer"]["right"]["rank"]
        for s in build_from_config_dict(bare).tensor_specs():
            assert all(want in (-1, got) for want, got in zip(s.shape, shapes[s.name])), s.name
            assert (-1 in s.shape) == (s.name.endswith(".a1") or s.name.endswith(".a2"))


@pytest.mark.parametrize("window,keep", [(100, 5), (100, 70), (1, 64), (64, 65), (30, 200)])
def test_a_decode_step_over_a_window_and_kept_tokens_lists_their_pages(window, keep):
    """The work list of a group that keeps first tokens beside a window: the pages of the first tokens,
    then those of the window, each once, in runs of the step's length; in the block that stays in place."""
    e = host_engine(max_tokens=64 * 64, max_seq_len=1024, n_slots=3, layers=2, windows=(0, window), v_head_dim=16, keep_first=keep)
    lengths = [500, 3, 130]
    slots = [e.slot_alloc() for _ in range(3)]
    for lo in range(0, 500, 250):
        live = [i for i in range(3) if lengths[i] > lo]
        e.step([slots[i] for i in live], [[1] * min(250, lengths[i] - lo) for i in live])
    for step in range(150):
        pos = [n + step for n in lengths]
        e.step(slots, [[7]] * 3)
        ppc = decode_pages_per_chunk(pos, G, 16)
        got = e.step_array("chunks.1").reshape(-1, 8)
        got = got[1:1 + got[0, 0]].tolist()
        want = []
        for i, p in enumerate(pos):
            first = max(0, p - window + 1) // 64                       # whole pages, so a kept page may hold a few more tokens
            seen = [j for j in range(p // 64 + 1) if j >= first or j < (keep + 63) // 64]
            table = e.slot_pages(1, slots[i])
            for c in range(0, len(seen), ppc):
                pages = [int(table[j]) for j in seen[c:c + ppc]][:4]
                want.append([i, c // ppc, p, slots[i]] + pages + [-1] * (4 - len(pages)))
        assert sorted(got) == sorted(want), step


def test_kept_tokens_need_a_window_and_a_group_that_keeps_every_key():
    with pytest.raises(Exception) as e:
        host_engine(windows=(0,), keep_first=3, v_head_dim=16, all_groups=True)
    assert "keeps 3 first tokens" in str(e.value)


# ------------------------------------------------------------------------------ closed forms of the plain model
def test_the_plain_norm_has_eps_inside_the_root_and_a_plain_weight():
    x = np.array([[1.0, 2.0, 3.0, 6.0]])
    w = np.array([1.0, 2.0, 0.5, 0.0])
    assert np.allclose(P.rms_norm(x, w, 0.5), x / math.sqrt(12.5 + 0.5) * w)
    assert np.allclose(P.unit_rms(x, 3.5), x / 4.0)


def test_the_plain_rotation_turns_adjacent_entries():
    rot = dict(base=100.0, dims=4)
    x = np.array([[[1.0, 2.0, 3.0, 4.0, 9.0]]])                       # one token, one head; the fifth entry is not turned
    a0, a1 = 3.0, 0.3
    assert np.allclose(P.rotate(x, rot, [3])[0, 0], [math.cos(a0) - 2 * math.sin(a0), 2 * math.cos(a0) + math.sin(a0),
                                                     3 * math.cos(a1) - 4 * math.sin(a1), 4 * math.cos(a1) + 3 * math.sin(a1), 9.0])
    assert np.allclose(P.rotate(x, rot, [0]), x)
    # base 4, eight entries: frequencies 1, 2^-1/2, 1/2, 2^-3/2, wavelengths 2 pi times 1, 2^1/2, 2, 2^3/2; the limits lie at
    # 2 pi 1.2 and 2 pi 2.4: the first keeps its pace, the last is slowed, the two between are blended
    rot = dict(base=4.0, dims=8, scaling=zt.slowed(5.0, 1.0, 2.0, 2 * math.pi * 2.4))
    f = 4.0 ** (-np.arange(4) / 4.0)
    s = 2.4 * f - 1.0
    want = [f[0], (1 - s[1]) * f[1] / 5 + s[1] * f[1], (1 - s[2]) * f[2] / 5 + s[2] * f[2], f[3] / 5]
    assert np.allclose(P.rotary_frequencies(rot), want, rtol=1e-12)


def test_the_product_side_frequencies_are_the_plain_ones():
    from picolm_amd.config.zalalix import RotationConfig
    from picolm_amd.parts.position import rotary_inv_freq
    for rot in (dict(base=4.0, dims=8, scaling=zt.slowed(5.0, 1.0, 2.0, 15.0)), dict(base=30000.0, dims=28, scaling=zt.slowed(3.0, 0.5, 7.0, 300)),
                dict(base=77.0, dims=6), dict(base=500.0, dims=32, scaling=zt.slowed(2.0, 1.0, 1.0, 100))):
        c = RotationConfig.from_dict(rot, "")
        assert np.allclose(rotary_inv_freq(c.dims, c.base, c.scaling).numpy(), P.rotary_frequencies(rot), rtol=1e-12)


def test_the_plain_mask_cap_and_softmax():
    mask = dict(size=3, keep_first=2)
    assert [j for j in range(9) if P.sees(7, j, mask)] == [0, 1, 5, 6, 7]
    assert [j for j in range(9) if P.sees(2, j, mask)] == [0, 1, 2] and [j for j in range(9) if P.sees(0, j, mask)] == [0]
    assert np.allclose(P.capped(np.array([1e-6, 100.0, -100.0]), 5.0), [1e-6, 5.0, -5.0])
    q = np.array([[[1.0, 0.0]], [[1.0, 0.0]]])                        # two tokens, one head
    k = np.array([[[math.log(2.0), 0.0]], [[math.log(3.0), 0.0]]])
    v = np.array([[[1.0, 0.0]], [[0.0, 1.0]]])
    wide = dict(size=9, keep_first=0)
    assert np.allclose(P.softmax_attention(q, k, v, 1.0, 1e6, wide)[1, 0], [2 / 6, 3 / 6])
    assert np.allclose(P.softmax_attention(q, k, v, 1.0, 1e6, wide)[0, 0], [2 / 3, 0.0])
    assert np.allclose(P.softmax_attention(q, -1000 * k, v, 1.0, 1e6, wide)[1, 0], [0.0, 0.0])
    assert np.allclose(P.softmax_attention(q, 1000 * k, v, 1.0, math.log(4.0), wide)[1, 0], [4 / 9, 4 / 9])     # both scores at the cap
    assert np.allclose(P.softmax_attention(q, k, v, 1.0, 1e6, dict(size=1, keep_first=0))[1, 0], [0.0, 3 / 4])
    # grouped heads: query heads 0, 1 read KV head 0, heads 2, 3 read KV head 1
    v2 = np.array([[[1.0, 2.0], [3.0, 4.0]]])
    assert np.allclose(P.softmax_attention(np.zeros((1, 4, 2)), np.ones((1, 2, 2)), v2, 1.0, 9.0, wide)[0], np.array([[1, 2], [1, 2], [3, 4], [3, 4]]) / 2)


def test_the_plain_state_decays_before_it_takes_the_token_and_is_read_after():
    q, k, v = np.array([[[1.0, 2.0]], [[3.0, 1.0]]]), np.array([[[1.0, 0.0]], [[2.0, 5.0]]]), np.array([[[7.0]], [[11.0]]])
    decay = np.array([[[9.0, 9.0]], [[0.5, 0.25]]])                    # the first token's decay meets a state of zeros
    out = P.decayed_state_walk(q, k, v, decay)
    assert np.allclose(out[:, 0, 0], [7.0, 3.0 * (0.5 * 7 + 2 * 11) + 1.0 * (5 * 11)])


def one_layer(mixer, ff=None, width=16, **kw):
    return zt.config(50, width, [zt.layer(mixer, ff)], **kw)


def test_the_plain_lightning_and_retention_of_two_tokens():
    rng = np.random.default_rng(0)
    h = rng.normal(size=(2, 16))
    for kind in ("lightning", "retention"):
        mixer = (zt.lightning if kind == "lightning" else zt.retention)(4, 6, [0.5, 0.25])
        W = zt.as_arrays(zt.make_weights(one_layer(mixer), 3))
        p = "l0.mix."
        f = P.silu if kind == "lightning" else (lambda z: z)
        q, k, v = (f(h @ W[p + n].T).reshape(2, 2, -1) for n in "qkv")
        if kind == "retention":
            k = k / 2.0                                                # 4^(-1/2)
        o = np.stack([0.0 * v[1] + d * (q[1, a] @ k[0, a]) * v[0, a] * np.eye(2)[a][:, None] for a, d in enumerate((0.5, 0.25))]).sum(0)
        o = o + np.stack([(q[1, a] @ k[1, a]) * v[1, a] for a in range(2)])
        g = h[1] @ W[p + "g"].T
        if kind == "lightning":
            flat = o.reshape(-1)
            y = flat / np.sqrt((flat ** 2).mean() + 1e-6) * W[p + "norm"] / (1 + np.exp(-g))
        else:
            y = (o / np.sqrt((o ** 2).mean(1, keepdims=True) + 1e-6)).reshape(-1) * g / (1 + np.exp(-g))
        got = P.MIXERS[kind](h, W, p, mixer[1], 1e-6)
        assert np.allclose(got[1], W[p + "o"] @ y), kind


def test_the_plain_channel_decays_and_gated_linear_attention():
    m = zt.gla(2, 4, 6, 2.0, 3)
    cfg = one_layer(zt.parallel(zt.windowed(2, 1, 4, 6, 0.5, 4, 1, zt.rotation(2)), m))
    W = zt.as_arrays(zt.make_weights(cfg, 5))
    p = "l0.mix.right."
    h = np.random.default_rng(1).normal(size=(2, 16))
    z = h @ W[p + "a1"].T @ W[p + "a2"].T + W[p + "a2.b"]
    a = P.channel_decays(h, W, p, m)
    assert np.allclose(a.reshape(2, 8), np.sqrt(1 / (1 + np.exp(-z)))) and a.shape == (2, 2, 4)
    q, k, v = (h @ W[p + n].T for n in "qkv")
    o = []
    for n in range(2):
        s, t = slice(4 * n, 4 * n + 4), slice(6 * n, 6 * n + 6)
        S = np.diag(a[1, n]) @ np.outer(k[0, s], v[0, t]) + np.outer(k[1, s], v[1, t])
        y = S.T @ (q[1, s] / 2.0)
        o.append(y / np.sqrt((y ** 2).mean() + 1e-6) * W[p + "norm"])
    g = h[1] @ W[p + "g"].T
    assert np.allclose(P.gated_linear_attention(h, W, p, m, 1e-6)[1], W[p + "o"] @ (np.concatenate(o) * g / (1 + np.exp(-g))))


def test_the_plain_windowed_attention_of_one_token_and_the_sum_of_branches():
    left = zt.windowed(4, 2, 6, 5, 0.5, 3, 1, zt.rotation(4, 10.0), 3.0)
    cfg = one_layer(zt.parallel(left, zt.gla(1, 4, 6, 2.0, 3), 0.5, -2.0))
    W = zt.as_arrays(zt.make_weights(cfg, 7))
    p = "l0.mix.left."
    h = np.random.default_rng(2).normal(size=(1, 16))
    q, k, v = (h[0] @ W[p + n].T + W[p + n + ".b"] for n in "qkv")
    q = q / np.sqrt((q ** 2).mean() + 1e-6) * W[p + "q.norm"]         # one norm over the four heads of 6, one over the two of k
    k = k / np.sqrt((k ** 2).mean() + 1e-6) * W[p + "k.norm"]
    out = []
    for n in range(4):                                                # position 0: nothing turns
        s = 3.0 * math.tanh(0.5 * q[6 * n:6 * n + 6] @ k[6 * (n // 2):6 * (n // 2) + 6] / 3.0)
        gate = 1 / (1 + math.exp(-(h[0] @ W[p + "g"][n])))
        out.append(v[5 * (n // 2):5 * (n // 2) + 5] * math.exp(s) / (1 + math.exp(s)) * gate)
    want = W[p + "o"] @ np.concatenate(out) + W[p + "o.b"]
    got = P.windowed_attention(h, W, p, left, 1e-6)
    assert np.allclose(got[0], want)
    right = P.gated_linear_attention(h, W, "l0.mix.right.", cfg["layers"][0]["mixer"]["right"], 1e-6)
    assert np.allclose(P.parallel(h, W, "l0.mix.", cfg["layers"][0]["mixer"], 1e-6), 0.5 * got - 2.0 * right)


def test_every_tensor_and_constant_shows_in_the_plain_logits():
    cfg = zt.CONFIG_A
    w = zt.make_weights(cfg, 0)
    tokens = [int(t) for t in np.random.default_rng(0).integers(0, cfg["vocab"], size=60)]
    base = zt.plain_logits(cfg, w, tokens)
    for name, t in w.items():
        changed = dict(w)
        changed[name] = (t.double() * 1.3 + 0.1 * torch.arange(t.numel(), dtype=torch.float64).reshape(t.shape).remainder(7)).to(torch.bfloat16)
        # (the logits' common part is taken off: a change of the head that every row shares would not show)
        assert zt.distance(zt.plain_logits(cfg, changed, tokens), base) > 1e-4, name
    for path, value in [(("embedding", "scale"), 5.0), (("norm", "eps"), 0.3), (LEFT + ("scale",), 0.5), (LEFT + ("softcap",), 0.7),
                        (LEFT + ("mask", "size"), 20), (LEFT + ("mask", "keep_first"), 2), (LEFT + ("rot", "base"), 100.0),
                        (LEFT + ("rot", "dims"), 4), (LEFT + ("rot", "scaling", "factor"), 9.0), (LEFT + ("rot", "scaling", "low"), 0.3),
                        (LEFT + ("rot", "scaling", "high"), 9.0), (LEFT + ("rot", "scaling", "original"), 20),
                        (("layers", 0, "mixer", "left_scale"), 0.2), (("layers", 0, "mixer", "right_scale"), 0.2), (RIGHT + ("tau",), 1.0),
                        (("layers", 1, "mixer", "decay", 0), 0.5), (("layers", 2, "mixer", "decay", 2), 0.9)]:
        other = copy.deepcopy(cfg)
        at = other
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        assert zt.distance(zt.plain_logits(other, w, tokens), base) > 1e-4, path
