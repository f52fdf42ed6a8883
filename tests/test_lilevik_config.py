"""The Lilevik configuration without a GPU: keys and errors, tensor names and shapes against the plain implementation's, what
reaches the parts, the stretched frequencies, the pages that a chunk gives back, and properties of the plain implementation
itself."""
import copy
import math

import pytest
import torch

import plain_lilevik as P
from rbitnet_amd.cache.pages import PAGE_SIZE, PageTable
from rbitnet_amd.config import load_config
from rbitnet_amd.engine.model import expected_tensors
from rbitnet_amd.errors import ConfigError
from rbitnet_amd.parts.position import rope_amplitude, rope_inverse_frequencies


def latent(heads=3, dim=8, rot_dim=4, vdim=6, q_rank=12, kv_rank=10, scale=0.3, base=100.0):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale,
                rot={"base": base, "dims": rot_dim})


def attention(heads=4, kv_heads=2, dim=8, vdim=6, dims=4, base=50.0, scale=0.35, chunk=5, scaling=None):
    out = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot={"base": base, "dims": dims})
    if scaling:
        out["rot"]["scaling"] = scaling
    if chunk:
        out["mask"] = {"size": chunk}
    return out


def moe(ff=20, experts=5, top=2):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


YARN = {"factor": 4.0, "original": 64, "fast": 32.0, "slow": 1.0}
CFG = {"architecture": "Lilevik", "vocab": 40, "width": 24, "norm": {"eps": 1e-5}, "layers": [
    {"type": "lightning", "mixer": dict(heads=2, dim=8, vdim=12, decay=[0.5, 0.99]), "mlp": moe()},
    {"type": "attention", "mixer": attention(scaling=YARN), "mlp": None},
    {"type": "latent_attention", "mixer": latent(), "mlp": moe(12, 3, 3)},
    {"type": "attention", "mixer": attention(heads=3, kv_heads=3, vdim=10, dims=0, chunk=None), "mlp": moe(8, 4, 1)}]}


def test_tensor_names_and_shapes_are_the_plain_implementations():
    cfg, spec = load_config(copy.deepcopy(CFG))
    got = {k: tuple(v.shape) for k, v in expected_tensors(spec).items()}
    assert got == P.tensor_shapes(CFG)
    assert cfg.to_dict() == CFG and load_config(cfg.to_dict())[0] == cfg


def test_the_order_of_layers_and_the_choices_reach_the_parts():
    _, spec = load_config(copy.deepcopy(CFG))
    assert [l.mixer.kind for l in spec.layers] == ["lightning", "attention", "latent_attention", "attention"]
    assert all(l.block == "sandwich" for l in spec.layers) and spec.layers[1].feed_forward is None
    assert spec.layers[0].mixer["decay"] == [0.5, 0.99]
    a, last = spec.layers[1].mixer, spec.layers[3].mixer
    assert a["chunk"] == 5 and a["weights"] == "sigmoid" and a["qk_norm"]["over"] == "projection" and a["value_norm"] == 1e-5
    assert a["position"].params["style"] == "interleaved" and a["position"].params["scaling"]["rope_type"] == "yarn"
    assert last["chunk"] is None and last["position"].kind == "none"
    lat = spec.layers[2].mixer
    assert lat["position"].params["style"] == "interleaved" and not lat["sink"] and not lat["head_gate"]
    ff = spec.layers[2].feed_forward
    assert (ff["experts"], ff["top"], ff["intermediate_size"], ff["score"], ff["bias"], ff["weight_on"]) == (3, 3, 12, "chosen", True, "output")
    assert spec.head["name"] is None and spec.embedding["name"] == "embed"


@pytest.mark.parametrize("edit,match", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="delta"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, "x"]), "decay"),
    (lambda c: c["layers"][0]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "share"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("fast"), "fast"),
    (lambda c: c["layers"][1]["mixer"]["rot"].pop("base"), "base"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"]["mask"].pop("size"), "size"),
    (lambda c: c["layers"][2]["mixer"].update(rot={"base": 10.0, "dims": 2}), "rot"),
    (lambda c: c["layers"][2]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "moe"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "top"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("ff"), "ff"),
])
def test_errors_name_the_key(edit, match):
    raw = copy.deepcopy(CFG)
    edit(raw)
    with pytest.raises(ConfigError, match=match):
        load_config(raw)


@pytest.mark.parametrize("dims,base,scaling", [
    (24, 3e4, {"factor": 5.0, "original": 900, "fast": 24.0, "slow": 1.5}),
    (64, 1e4, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
    (4, 10.0, {"factor": 2.0, "original": 8, "fast": 4.0, "slow": 0.5}),
    (2, 100.0, {"factor": 3.0, "original": 50, "fast": 1.0, "slow": 1.0}),
    (16, 1e6, {"factor": 16.0, "original": 100000, "fast": 2.0, "slow": 1.5}),
    (8, 1e4, {"factor": 1.0, "original": 64, "fast": 32.0, "slow": 1.0}),
])
def test_stretched_frequencies(dims, base, scaling):
    f, m = P.frequencies(dims, base, scaling)
    s = dict(scaling, rope_type="yarn")
    assert torch.allclose(rope_inverse_frequencies(dims, base, s), f, rtol=1e-12, atol=0)
    assert abs(rope_amplitude(s) - m) < 1e-12 and rope_amplitude(None) == 1.0
    plain, one = P.frequencies(dims, base)
    assert one == 1.0 and torch.all(f <= plain * (1 + 1e-12)) and torch.all(f >= plain / scaling["factor"] * (1 - 1e-12))


def test_a_ramp_by_hand():
    # eight pairs, base e^8: pair i turns original / (2 pi e^i) times; 5 pi turns at index ln(original / (10 pi^2)), and so on
    dims, base = 16, math.exp(16.0)
    original = 2.0 * math.pi * math.exp(6.0)
    f, m = P.frequencies(dims, base, {"factor": 10.0, "original": original, "fast": math.exp(3.5), "slow": math.exp(1.5)})
    # index(t) = 16 (6 - ln t) / 32: fast 1.25 -> lo 1, slow 2.25 -> hi 3
    plain = [base ** (-2.0 * i / dims) for i in range(8)]
    want = [plain[0], plain[1], 0.55 * plain[2]] + [x / 10.0 for x in plain[3:]]
    assert torch.allclose(f, torch.tensor(want, dtype=torch.float64), rtol=1e-9)
    assert abs(m - (0.1 * math.log(10.0) + 1.0)) < 1e-12


def test_a_chunk_gives_pages_back():
    from rbitnet_amd.config.spec import PartSpec
    from rbitnet_amd.parts import BuildEnv, build_part
    _, spec = load_config(copy.deepcopy(CFG))
    env = BuildEnv(hidden_size=24, dtype=torch.float32, device=torch.device("cpu"), lib=None)
    assert build_part("mixer", spec.layers[1].mixer, env).cache_request().window == 5
    assert build_part("mixer", spec.layers[3].mixer, env).cache_request().window is None
    # a window as long as the chunk never gives back what the chunk's queries still see
    for chunk in (5, 64, 70, 200):
        t = PageTable(40, window=chunk)
        t.open(0)
        for length in range(1, 600, 7):
            t.ensure(0, length)
            t.release_behind(0, length)
            first = length // chunk * chunk                       # the next query's chunk begins here
            assert all(p >= 0 for p in t.pages(0)[first // PAGE_SIZE:]), (chunk, length)
        assert t.pages(0)[0] < 0 or chunk >= 600
        t.check()


def test_the_plain_implementations_own_properties():
    # a chunk as long as the sequence is plain causal sight; a chunk of one is the token alone
    assert torch.equal(P.visible(6, 6), P.visible(6)) and torch.equal(P.visible(5, 1), torch.eye(5, dtype=torch.bool))
    assert P.visible(9, 4)[6].tolist() == [False] * 4 + [True] * 3 + [False] * 2
    # a rotation by position keeps scores a function of the distance, and lengths up to the factor
    f, m = P.frequencies(8, 100.0, YARN)
    x = torch.randn(1, 1, 10, dtype=torch.float64)
    a, b = P.rotate(x, f, m, 7), P.rotate(x.flip(-1), f, m, 4)
    c, d = P.rotate(x, f, m, 107), P.rotate(x.flip(-1), f, m, 104)
    assert torch.allclose((a * b).sum(), (c * d).sum(), atol=1e-10)
    assert torch.allclose(a[..., :8].norm(), m * x[..., :8].norm()) and torch.equal(a[..., 8:], x[..., 8:])
    # the decaying sum written out
    q, k, v = (torch.randn(7, 2, n, dtype=torch.float64) for n in (3, 3, 4))
    decay = torch.tensor([0.5, 1.0], dtype=torch.float64)
    i, j = torch.arange(7)[:, None], torch.arange(7)[None, :]
    w = torch.stack([(q[:, h] @ k[:, h].T) * torch.where(j <= i, decay[h] ** (i - j).clamp(min=0), torch.zeros((), dtype=torch.float64))
                     for h in range(2)])
    assert torch.allclose(P.decaying_sum(q, k, v, decay), torch.einsum("hij,jhd->ihd", w, v), atol=1e-12)
    # weights over the chosen sum to one, and a chosen one's weight does not depend on the others' logits
    h = torch.randn(11, 6, dtype=torch.float64)
    r, bias = torch.randn(5, 6, dtype=torch.float64), torch.randn(5, dtype=torch.float64)
    chosen, weights = P.route(h, r, bias, 3)
    assert torch.allclose(weights.sum(-1), torch.ones(11, dtype=torch.float64)) and int(chosen.max()) < 5
