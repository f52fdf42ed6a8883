"""The Goperax configuration without a GPU: keys and errors, tensor names and shapes against the plain implementation's, the order
of layers with a loop, what reaches the parts, what the cache keeps, and properties of the plain implementation itself."""
import copy
import math

import pytest
import torch

import plain_goperax as P
from rbitnet_amd.config import load_config
from rbitnet_amd.config.spec import PartSpec
from rbitnet_amd.engine.model import expected_tensors
from rbitnet_amd.errors import ConfigError
from rbitnet_amd.parts import BuildEnv, build_part


def scan(heads=4, vdim=6, state=10, groups=2, conv=3, norm_groups=3):
    return dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


def soft(heads=4, kv_heads=2, dim=8, scale=0.3, cap=20.0, window=5):
    out = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale)
    if cap:
        out["softcap"] = cap
    if window:
        out["mask"] = {"size": window}
    return out


def moe(ff=20, experts=5, top=2, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


CFG = {"architecture": "Goperax", "vocab": 40, "width": 24, "streams": 3, "embedding": {"scale": 4.5}, "norm": {"eps": 1e-5},
       "loop": {"start": 1, "stop": 3, "times": 3}, "layers": [
           {"type": "mamba2", "mixer": scan(), "mlp": {"kind": "dense", "ff": 30}},
           {"type": "attention", "mixer": soft(), "mlp": None},
           {"type": "mamba2", "mixer": scan(3, 4, 6, 1, 1, 1), "mlp": moe(shared=12)},
           {"type": "attention", "mixer": soft(heads=3, kv_heads=3, cap=None, window=None), "mlp": moe(8, 4, 1)}]}


def test_tensor_names_and_shapes_are_the_plain_implementations():
    cfg, spec = load_config(copy.deepcopy(CFG))
    got = {k: tuple(v.shape) for k, v in expected_tensors(spec).items()}
    assert got == P.tensor_shapes(CFG)
    assert cfg.to_dict() == CFG and load_config(cfg.to_dict())[0] == cfg
    # a layer without a feed-forward has neither its norm nor its mixture; a file may hold them
    assert "l1.norm2" not in got and "l1.hc2.mix" not in got and {"l1.norm2", "l1.hc2.mix"} <= set(spec.optional_tensors)


@pytest.mark.parametrize("loop,want", [(None, [0, 1, 2, 3]), ({"start": 1, "stop": 3, "times": 3}, [0, 1, 2, 1, 2, 1, 2, 3]),
                                       ({"start": 0, "stop": 4, "times": 2}, [0, 1, 2, 3] * 2), ({"start": 3, "stop": 4, "times": 1}, [0, 1, 2, 3]),
                                       ({"start": 0, "stop": 1, "times": 4}, [0, 0, 0, 0, 1, 2, 3])])
def test_the_order_of_layers(loop, want):
    raw = dict(copy.deepcopy(CFG), loop=loop)
    _, spec = load_config(raw)
    assert spec.schedule == want == P.run_order(raw)
    raw.pop("loop")
    if loop is None:
        assert load_config(raw)[1].schedule == want


def test_the_choices_reach_the_parts():
    _, spec = load_config(copy.deepcopy(CFG))
    assert [l.mixer.kind for l in spec.layers] == ["state_space", "attention", "state_space", "attention"]
    assert all(l.block == "hyper" and l.params == {"streams": 3, "scale": False} for l in spec.layers)
    assert spec.layers[0].mixer.params == dict(scan(), eps=1e-5)
    a, last = spec.layers[1].mixer, spec.layers[3].mixer
    assert (a["window"], a["softcap"], a["values"], a["sink"], a["position"].kind) == (5, 20.0, "keys", "one", "none")
    assert last["window"] is None and last["softcap"] is None
    ff = spec.layers[2].feed_forward
    assert (ff["score"], ff["unit"], ff["weight_on"], ff["shared"]) == ("chosen", "squared_relu", "output", {"intermediate_size": 12, "gate": False})
    assert spec.layers[3].feed_forward["shared"] is None and spec.layers[0].feed_forward["activation"] == "squared_relu"
    assert spec.embedding["scale"] == 4.5 and spec.embedding["waves"] == 10000.0 and spec.embedding["streams"] == 3
    assert spec.head["name"] is None


@pytest.mark.parametrize("edit,match", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.update(streams=0), "streams"),
    (lambda c: c["embedding"].pop("scale"), "scale"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="mamba"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), "share"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), "equal parts"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "share"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=6), "vdim"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][1]["mixer"]["mask"].pop("size"), "size"),
    (lambda c: c["layers"][0]["mlp"].update(kind="glu"), "dense"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda c: c["layers"][2]["mlp"]["router"].update(top=6), "top"),
    (lambda c: c["layers"][2]["mlp"]["shared"].pop("ff"), "shared"),
    (lambda c: c["loop"].update(stop=5), "loop"),
    (lambda c: c["loop"].update(start=3), "loop"),
    (lambda c: c["loop"].pop("times"), "times"),
])
def test_errors_name_the_key(edit, match):
    raw = copy.deepcopy(CFG)
    edit(raw)
    with pytest.raises(ConfigError, match=match):
        load_config(raw)


def test_what_the_cache_keeps():
    """One set of pages that are keys and values at once; a state and the convolution's inputs per sequence, and nothing of the
    convolution where it has one tap; a place of its own for every pass of a loop."""
    from rbitnet_amd.cache import Cache
    from rbitnet_amd.engine.model import Model
    _, spec = load_config(copy.deepcopy(CFG))
    env = BuildEnv(hidden_size=24, dtype=torch.float32, device=torch.device("cpu"), lib=None)
    first, att, bare, last = (build_part("mixer", l.mixer, env) for l in spec.layers)
    assert [(r.name, r.state_shape) for r in first.cache_requests()] == [("scan", (4, 6, 10)), ("conv", (2, 4 * 6 + 2 * 2 * 10))]
    assert [(r.name, r.state_shape) for r in bare.cache_requests()] == [("scan", (3, 4, 6))]
    (r,) = att.cache_requests()
    assert not r.values and r.window == 5 and (r.heads, r.head_dim) == (2, 8)
    assert last.cache_requests()[0].window is None
    model = Model(spec, torch.float32, "cpu", None)
    cache = Cache(model.cache_requests(), 2, 128, torch.float32, "cpu")
    assert len(cache.layer_groups) == len(spec.schedule) == 8
    slot = cache.alloc_slot()
    tables = {id(g): torch.zeros(1, 1, dtype=torch.int32) for g in cache.kv_groups}
    views = [cache.view(place, tables) for place in range(8)]
    assert views[1].v_pages.data_ptr() == views[1].k_pages.data_ptr()
    assert len({views[p].k_pages.data_ptr() for p in (1, 3, 5)}) == 3 and len({views[p].states["scan"].data_ptr() for p in (2, 4, 6)}) == 3
    cache.free_slot(slot)


@pytest.mark.parametrize("params,match", [
    ({"values": "keys", "value_dim": 6}, "values that are the keys"), ({"values": "keys", "conv": 3}, "values that are the keys"),
    ({"values": "keys", "cache_from": 0}, "values that are the keys"), ({"values": "queries"}, "unknown values")])
def test_attention_refuses_what_does_not_go_with_shared_keys(params, match):
    env = BuildEnv(hidden_size=24, dtype=torch.float32, device=torch.device("cpu"), lib=None)
    base = {"num_heads": 2, "num_kv_heads": 1, "head_dim": 8, "scale": 1.0, "position": PartSpec("none", {})}
    with pytest.raises(ConfigError, match=match):
        build_part("mixer", PartSpec("attention", dict(base, **params)), env)


def test_a_stream_in_copies_refuses_other_norms():
    from rbitnet_amd.config.spec import LayerSpec
    from rbitnet_amd.parts.hyper import HyperBlock
    env = BuildEnv(hidden_size=24, dtype=torch.float32, device=torch.device("cpu"), lib=None)
    def layer(norm, **params):
        return LayerSpec(prefix="l", block="hyper", mixer=PartSpec("state_space", dict(scan(), eps=1e-5)), feed_forward=None, norm1=norm,
                         norm2=None, params=dict({"streams": 2}, **params))
    HyperBlock(layer(PartSpec("rmsnorm", {"size": 24, "eps": 1e-5}), scale=False), env)
    HyperBlock(layer(PartSpec("layernorm", {"size": 24, "eps": 1e-5})), env)
    with pytest.raises(ConfigError, match="norms that read such streams"):
        HyperBlock(layer(PartSpec("tanh", {"size": 24})), env)
    with pytest.raises(ConfigError, match="goes with layer norms"):
        HyperBlock(layer(PartSpec("rmsnorm", {"size": 24, "eps": 1e-5})), env)


def test_the_plain_implementations_own_properties():
    # the window: itself and the size - 1 tokens before it
    assert P.visible(9, 3)[6].tolist() == [False] * 4 + [True] * 3 + [False] * 2 and torch.equal(P.visible(5, 9), P.visible(5))
    assert torch.equal(P.visible(4, 1), torch.eye(4, dtype=torch.bool))
    # one beside the sum: a lone key of score 0 has half the weight, and large scores change nothing
    assert P.weights_beside_one(torch.zeros(1, 1, 1, dtype=torch.float64), P.visible(1)).item() == 0.5
    big = P.weights_beside_one(torch.full((1, 2, 2), 900.0, dtype=torch.float64), P.visible(2))
    assert torch.allclose(big[0], torch.tensor([[1.0, 0.0], [0.5, 0.5]], dtype=torch.float64))
    s = torch.randn(2, 6, 6, dtype=torch.float64)
    a, seen = P.weights_beside_one(s, P.visible(6, 4)), P.visible(6, 4).to(torch.float64)
    assert torch.allclose(a, s.exp() * seen / (1 + (s.exp() * seen).sum(-1, keepdim=True)))
    # the scan written out: y_i = sum_j dt_j exp(-rate sum_(j < t <= i) dt_t) (c_i . b_j) x_j + d x_i
    x, b, c = (torch.randn(7, n, m, dtype=torch.float64) for n, m in ((4, 3), (2, 5), (2, 5)))
    dt, a_log, d = torch.rand(7, 4, dtype=torch.float64), torch.randn(4, dtype=torch.float64), torch.randn(4, dtype=torch.float64)
    y = P.selective_scan(x, b, c, dt, a_log, d)
    for h in range(4):
        for i in range(7):
            want = d[h] * x[i, h]
            for j in range(i + 1):
                want = want + dt[j, h] * math.exp(-math.exp(a_log[h]) * float(dt[j + 1:i + 1, h].sum())) * (c[i, h // 2] @ b[j, h // 2]) * x[j, h]
            assert torch.allclose(y[i, h], want, atol=1e-12)
    # the convolution's last tap is the current token's, and it starts from zeros
    taps, bias = torch.randn(3, 4, dtype=torch.float64), torch.randn(3, dtype=torch.float64)
    z = torch.randn(6, 3, dtype=torch.float64)
    out = P.causal_conv(z, taps, bias)
    assert torch.allclose(out[0], taps[:, 3] * z[0] + bias) and torch.allclose(out[1], taps[:, 3] * z[1] + taps[:, 2] * z[0] + bias)
    # the norm in parts gives every part unit mean square, the gate comes first
    g = P.gated_group_norm(torch.randn(5, 12, dtype=torch.float64), torch.randn(5, 12, dtype=torch.float64), torch.ones(12, dtype=torch.float64), 3, 0.0)
    assert torch.allclose((g.view(5, 3, 4) ** 2).mean(-1), torch.ones(5, 3, dtype=torch.float64))
    # weights of the chosen are the softmax over the chosen logits
    h, r = torch.randn(11, 6, dtype=torch.float64), torch.randn(5, 6, dtype=torch.float64)
    chosen, weights = P.route(h, r, 3)
    assert torch.allclose(weights, torch.softmax((h @ r.T).gather(1, chosen), -1))
    # copies: with one of them and all coefficients one, the plain residual sum
    one = torch.ones(1, dtype=torch.float64)
    assert torch.equal(P.rebuild_copies([z], one, one.view(1, 1), out)[0], z + out) and torch.equal(P.gather_copies([z], one), z)
    m = torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=torch.float64)
    new = P.rebuild_copies([z, out], torch.zeros(2, dtype=torch.float64), m, z)
    assert torch.allclose(new[1], 2 * z + 4 * out)
    # the sines and cosines of a position
    v = P.wave_vector(torch.tensor([3]), 5)
    assert torch.allclose(v[0], torch.tensor([math.sin(3), math.cos(3), math.sin(3 * 1e4 ** -0.4), math.cos(3 * 1e4 ** -0.4), math.sin(3 * 1e4 ** -0.8)],
                                             dtype=torch.float64))
