"""The Pinirax architecture without a GPU: its configuration, the model's tensors and what a request keeps, the layout of the
recurrences' state, and the plain statement's own mechanisms against hand-made cases."""
import copy
import math

import pytest
import torch

import plain_pinirax as pp
from ginfer_amd import config_from_dict
from ginfer_amd.cache import CacheManager
from ginfer_amd.config import ConfigError
from ginfer_amd.parts import KVCacheSpec, StateSpec
from ginfer_amd.parts.model import build_model

F64 = torch.float64


def LEFT(heads, kv_heads, dim, vdim, scale, size=None, cap=20.0):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if size is not None:
        m["mask"] = dict(size=size)
    if cap is not None:
        m["softcap"] = cap
    return m


def RIGHT(heads, kv_heads, dim, vdim, conv):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def PAR(left, right, left_scale=1.0, right_scale=1.0):
    return "parallel", dict(left=left, right=right, left_scale=left_scale, right_scale=right_scale)


def SSM(heads, vdim, state, groups, norm_groups, conv):
    return "mamba2", dict(heads=heads, vdim=vdim, state=state, groups=groups, norm_groups=norm_groups, conv=conv)


def MOE(experts, top, ff, identity=0):
    return dict(kind="moe", router=dict(experts=experts, top=top, identity=identity), expert=dict(ff=ff))


def config(width, vocab, layers, eps=1e-5, scale=2.0):
    """layers: (mixer, mlp) pairs, the mixer from PAR / SSM."""
    return dict(architecture="Pinirax", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=scale),
                layers=[dict(type=m[0], mixer=m[1], mlp=f) for m, f in layers])


CFG = config(48, 101, [
    (PAR(LEFT(4, 2, 12, 20, 0.3, size=9, cap=7.0), RIGHT(6, 3, 8, 12, 3), 0.7, 1.3), MOE(6, 2, 24, identity=2)),
    (SSM(6, 8, 20, 3, 4, 4), None),
    (PAR(LEFT(3, 1, 16, 8, 0.2, cap=None), RIGHT(2, 2, 20, 7, 1)), MOE(3, 3, 16)),
    (SSM(2, 12, 5, 1, 1, 1), MOE(1, 2, 8, identity=3)),
], eps=2e-6, scale=1.5)


def test_configuration_reads_every_size_and_round_trips():
    cfg = config_from_dict(CFG)
    assert type(cfg).__name__ == "PiniraxConfig" and cfg.to_dict() == CFG and config_from_dict(cfg.to_dict()) == cfg
    spec = cfg.model_spec()
    assert [l.arrangement for l in spec.layers] == ["sandwich"] * 4 and [e.layer for e in spec.schedule] == [0, 1, 2, 3]
    assert spec.embedding.kind == "sinusoidal_scaled" and spec.embedding.params["scale"] == 1.5 and not spec.head.params["tied"]
    m = spec.layers[0].parts["mixer"]
    assert m.kind == "parallel_sum" and m.params["scales"] == [0.7, 1.3] and m.params["names"] == ["left", "right"]
    left, right = m.params["branches"]
    p = left.params
    assert (p["num_heads"], p["num_kv_heads"], p["head_dim"], p["value_dim"], p["scale"], p["window"], p["soft_cap"], p["head_gate"]) == \
        (4, 2, 12, 20, 0.3, 9, 7.0, True)
    assert p["bias"] and not p["out_bias"] and p["head_norm_eps"] == 2e-6 and p["sink"] is None and p.get("position") is None
    p = right.params
    assert right.kind == "gated_delta" and (p["num_heads"], p["num_kv_heads"], p["key_dim"], p["value_dim"], p["taps"]) == (6, 3, 8, 12, 3)
    assert p["eps"] == 2e-6 and p["unit_eps"] == 1e-6
    p = spec.layers[1].parts["mixer"].params
    assert (p["num_heads"], p["value_dim"], p["state_size"], p["groups"], p["norm_groups"], p["taps"]) == (6, 8, 20, 3, 4, 4)
    f = spec.layers[0].parts["feed_forward"].params
    assert (f["num_experts"], f["identity"], f["top_k"], f["expert_size"], f["scoring"], f["correction"], f["normalise"], f["router_bias"]) == \
        (6, 2, 2, 24, "softmax", True, False, False)
    assert "feed_forward" not in spec.layers[1].parts and "feed_forward_out_norm" not in spec.layers[1].parts
    far = spec.layers[2].parts["mixer"].params["branches"][0].params
    assert far["window"] is None and far["soft_cap"] is None
    for role in ("mixer_norm", "mixer_out_norm"):
        assert spec.layers[0].parts[role].params["gain_offset"] == 1.0
    assert spec.final_norm.params["gain_offset"] == 1.0 and spec.final_norm.params["eps"] == 2e-6


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c["embedding"].update(scale="x"), "scale"),
    (lambda c: c["layers"][0].update(type="lstm"), "unknown mixer type"),
    (lambda c: c["layers"][0]["mixer"].pop("left"), "left"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(softcap=0), "softcap"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(kv_heads=4), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["right"].pop("conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c["layers"][1]["mixer"].update(groups=4), "multiple"),
    (lambda c: c["layers"][1]["mixer"].update(norm_groups=5), "norm_groups"),
    (lambda c: c["layers"][1]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "feed-forward kind"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "ff"),
    (lambda c: c["norm"].update(eps=0), "eps"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_configuration_errors_name_the_key(change, word):
    c = copy.deepcopy(CFG)
    change(c)
    with pytest.raises(ConfigError) as e:
        config_from_dict(c)
    assert word in str(e.value)


def test_tensor_names_shapes_and_what_a_request_keeps():
    model = build_model(config_from_dict(CFG).model_spec(), torch.bfloat16, torch.device("cpu"))
    specs = {n: tuple(s.shape) for n, s in model.weight_specs().items()}
    want = {"embed": (101, 48), "head": (101, 48), "final.norm": (48,)}
    for i in range(4):
        want.update({"l%d.norm1" % i: (48,), "l%d.norm1b" % i: (48,)})
        if i != 1:
            want.update({"l%d.norm2" % i: (48,), "l%d.norm2b" % i: (48,)})
    for i, E, I, F in ((0, 6, 2, 24), (2, 3, 0, 16), (3, 1, 3, 8)):
        want.update({"l%d.mlp.router" % i: (E + I, 48), "l%d.mlp.correction" % i: (E + I,)})
        for e in range(E):
            want.update({"l%d.mlp.e%d.gate" % (i, e): (F, 48), "l%d.mlp.e%d.up" % (i, e): (F, 48), "l%d.mlp.e%d.down" % (i, e): (48, F)})
    for i, (H, G, D, V), (h, g, d, v, t) in ((0, (4, 2, 12, 20), (6, 3, 8, 12, 3)), (2, (3, 1, 16, 8), (2, 2, 20, 7, 1))):
        p = "l%d.mix.left." % i
        want.update({p + "q": (H * D, 48), p + "k": (G * D, 48), p + "v": (G * V, 48), p + "q.b": (H * D,), p + "k.b": (G * D,), p + "v.b": (G * V,),
                     p + "q.norm": (D,), p + "k.norm": (D,), p + "g": (H, 48), p + "o": (48, H * V)})
        p = "l%d.mix.right." % i
        want.update({p + "q": (g * d, 48), p + "k": (g * d, 48), p + "v": (h * v, 48), p + "q.conv": (g * d, t), p + "k.conv": (g * d, t),
                     p + "v.conv": (h * v, t), p + "g": (h * v, 48), p + "b": (h, 48), p + "a": (h, 48), p + "A_log": (h,), p + "dt_bias": (h,),
                     p + "norm": (v,), p + "o": (48, h * v)})
    for i, H, V, N, G, t in ((1, 6, 8, 20, 3, 4), (3, 2, 12, 5, 1, 1)):
        p, inner = "l%d.mix." % i, H * V
        want.update({p + "in": (2 * inner + 2 * G * N + H, 48), p + "conv": (inner + 2 * G * N, t), p + "conv.b": (inner + 2 * G * N,),
                     p + "dt_bias": (H,), p + "A_log": (H,), p + "D": (H,), p + "norm": (inner,), p + "o": (48, inner)})
    assert specs == want
    caches = model.cache_specs()
    # the left mixer's pages (heads padded to 16), no convolution of its own; the right one's state and ring of inputs
    assert caches[0][0] is None and caches[0][1] == KVCacheSpec(2, 32, 9)
    assert caches[0][2] == StateSpec((6, 3, 1, 256), torch.float32) and caches[0][3] == StateSpec((3, 2 * 24 + 72), torch.float32)
    assert caches[2][1] == KVCacheSpec(1, 16, None) and caches[2][2] == StateSpec((2, 2, 1, 256), torch.float32) and caches[2][3] is None
    assert caches[1] == [StateSpec((6, 2, 1, 256), torch.float32), StateSpec((4, 48 + 120), torch.float32)]
    assert caches[3][1] is None and not CacheManager.supports_prefix_caching(caches)
    assert model.capturable()
    mods = model.kernel_modules()
    assert ("attention_mfma", {"HEAD_DIM": 32, "SOFT_CAP": 1}) in mods and ("attention_mfma", {"HEAD_DIM": 16}) in mods
    assert CacheManager.state_bytes(caches, 3) == 4 * 4 * (6 * 3 * 256 + 3 * 120 + 2 * 2 * 256 + 6 * 2 * 256 + 4 * 168 + 2 * 3 * 256)


def test_a_part_that_shares_products_joins_its_branches():
    """One matrix for both projections, one for both outputs, the branches' own ones gone."""
    cfg = config_from_dict(CFG)
    model = build_model(cfg.model_spec(), torch.float32, torch.device("cpu"))
    mixer = model.blocks[0].mixer
    g = torch.Generator().manual_seed(0)
    w = {n: torch.randn(s.shape, generator=g) for n, s in mixer.weight_specs().items()}
    mixer.bind_weights(w)
    rows = [w["left." + n] for n in ("q", "k", "v", "g")] + [w["right." + n] for n in ("q", "k", "v", "g", "b", "a")]
    assert torch.equal(mixer.w_in, torch.cat(rows))
    assert mixer.w_out.shape == (48, 4 * 32 + 72) and mixer.branches[0].w_qkv is None and mixer.branches[1].w_in is None
    o = mixer.w_out[:, :128].reshape(48, 4, 32)
    assert torch.equal(o[:, :, :20].reshape(48, 80), w["left.o"]) and not o[:, :, 20:].any()
    assert torch.equal(mixer.w_out[:, 128:], w["right.o"])
    odd = model.blocks[2].mixer                       # 3 * 16 + 14 columns: two of zeros behind them
    odd.bind_weights({n: torch.randn(s.shape, generator=g) for n, s in odd.weight_specs().items()})
    assert odd.w_out.shape == (48, 64) and not odd.w_out[:, 62:].any()


def test_identity_experts_belong_to_scores_of_every_expert():
    from ginfer_amd.parts.mlp import RoutedGLU
    kw = dict(dtype=torch.float32, device=None)
    with pytest.raises(ValueError):
        RoutedGLU(16, 4, 2, 8, identity=1, **kw)
    with pytest.raises(ValueError):
        RoutedGLU(16, 4, 2, 8, scoring="softmax", identity=1, shared_size=8, **kw)
    with pytest.raises(ValueError):
        RoutedGLU(16, 4, 6, 8, scoring="softmax", identity=1, **kw)
    part = RoutedGLU(16, 4, 5, 8, scoring="softmax", identity=1, router_bias=False, **kw)
    assert part.weight_specs()["router"].shape == (5, 16) and "e4.gate" not in part.weight_specs()


def test_the_states_layout_holds_every_element_once():
    from ginfer_amd.kernels import ops
    for heads, dim, vdim in ((1, 64, 4), (3, 128, 7), (2, 5, 1), (2, 200, 33)):
        shape = ops.delta_state_shape(heads, dim, vdim)
        s = torch.arange(math.prod(shape), dtype=torch.float64).reshape(shape)
        m = ops.delta_state_matrix(s, dim, vdim)
        assert m.shape == (heads, dim, vdim) and m.unique().numel() == m.numel()
        for h, i, c in ((0, 0, 0), (heads - 1, dim - 1, vdim - 1), (0, dim // 2, vdim // 2)):
            j, s16, k = i // 64, i % 64 // 4, i % 4
            lane = (c % 4) * 16 + s16
            assert m[h, i, c] == s[h, c // 4, j, lane * 4 + k]
        both = torch.stack([s, s + 0.5])
        assert torch.equal(ops.delta_state_matrix(both, dim, vdim)[1], m + 0.5)


def test_plain_mechanisms_on_hand_made_cases():
    # positions: the sine of 0 and the cosine of 0 at the start, the first pair turning by a radian a token
    p = pp.position_vectors(3, 4)
    assert torch.equal(p[0], torch.tensor([0.0, 1.0, 0.0, 1.0], dtype=F64))
    assert abs(float(p[2, 0]) - math.sin(2.0)) < 1e-12 and abs(float(p[2, 1]) - math.cos(2.0)) < 1e-12
    assert abs(float(p[1, 2]) - math.sin(0.01)) < 1e-9
    # a convolution: the last column is the current token's, zeros before the start
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=F64)
    y = pp.causal_convolution(x, torch.tensor([[3.0, 2.0, 1.0]], dtype=F64), torch.tensor([0.5], dtype=F64))
    assert torch.equal(y[:, 0], torch.tensor([1.5, 12.5, 123.5], dtype=F64))
    # the delta rule without decay and with b = 1 stores v under a unit k exactly, and overwrites it
    k = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]], [[0.0, 1.0]]], dtype=F64)
    v = torch.tensor([[[5.0]], [[7.0]], [[2.0]]], dtype=F64)
    one = torch.ones((3, 1), dtype=F64)
    o, S = pp.gated_delta_rule(k, k, v, one, one)
    assert torch.equal(o[:, 0, 0], torch.tensor([5.0, 7.0, 2.0], dtype=F64)) and torch.equal(S[0, :, 0], torch.tensor([7.0, 2.0], dtype=F64))
    # decay comes before the correction: half of what is stored is gone when the error is taken
    o, S = pp.gated_delta_rule(k[:2], k[:2], v[:2], 0.5 * one[:2], 0.5 * one[:2])
    assert torch.allclose(o[:, 0, 0], torch.tensor([2.5, 1.25 + 0.5 * (7.0 - 1.25)], dtype=F64))
    # the state space: what token 0 wrote decays, the skip adds the token's own input
    B = torch.tensor([[[1.0]], [[2.0]]], dtype=F64)
    y, S = pp.state_space(torch.tensor([[[3.0]], [[4.0]]], dtype=F64), B, torch.ones_like(B), torch.tensor([[0.5], [1.0]], dtype=F64),
                          torch.tensor([[0.9], [0.1]], dtype=F64), torch.tensor([10.0], dtype=F64))
    assert torch.allclose(y[:, 0, 0], torch.tensor([1.5 + 30.0, 0.15 + 8.0 + 40.0], dtype=F64))
    # a norm in parts: each part has its own root mean square
    y = pp.parts_norm(torch.tensor([[3.0, 3.0, 0.5, 0.5]], dtype=F64), 2, torch.ones(4, dtype=F64), 0.0)
    assert torch.allclose(y, torch.ones((1, 4), dtype=F64))
    # window: a query sees itself and size - 1 tokens before it; the cap bounds what one key can weigh
    q = torch.ones((4, 1, 1), dtype=F64)
    vals = torch.tensor([[[1.0]], [[10.0]], [[100.0]], [[1000.0]]], dtype=F64)
    o = pp.capped_window_attention(q, q, vals, 1.0, 5.0, 2)
    assert torch.allclose(o[:, 0, 0], torch.tensor([1.0, 5.5, 55.0, 550.0], dtype=F64))
    keys = torch.tensor([[[1000.0]], [[0.0]]], dtype=F64)
    o = pp.capped_window_attention(torch.ones((2, 1, 1), dtype=F64), keys, vals[:2], 1.0, 2.0, None)
    assert abs(float(o[1, 0, 0]) - (math.exp(2.0) + 10.0) / (math.exp(2.0) + 1.0)) < 1e-9
    # routing: the correction changes the choice and not the weight; an identity expert gives the row itself
    h = torch.tensor([[1.0, 2.0]], dtype=F64)
    w = {"router": torch.zeros((3, 2), dtype=F64), "correction": torch.tensor([0.0, 0.0, 1.0], dtype=F64)}
    for e in range(2):
        w.update({"e%d.gate" % e: torch.ones((1, 2), dtype=F64), "e%d.up" % e: torch.ones((1, 2), dtype=F64), "e%d.down" % e: torch.ones((2, 1), dtype=F64)})
    mlp = dict(router=dict(experts=2, identity=1, top=1))
    assert torch.allclose(pp.routed_feed_forward(h, w, "", mlp), h / 3.0)
    mlp["router"]["top"] = 2
    z = 3.0
    assert torch.allclose(pp.routed_feed_forward(h, w, "", mlp), h / 3.0 + z / (1 + math.exp(-z)) * z / 3.0)
