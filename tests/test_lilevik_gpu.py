"""The Lilevik parts and whole models on the GPU against the plain implementation of `plain_lilevik.py`: each mechanism
alone; a prompt whole, in pieces down to two tokens and token by token; batches of unequal requests against each alone;
slots and pages used again; keys far away, at page borders, just inside and just outside every chunk, in prompts and in
decoding; the first tokens of a sequence; long decoding; sizes that differ in everything (and values that a model may happen
to make equal or 1); greedy generation through `Engine.generate`.  Configurations and weights are made here."""
import copy
import io
import json
import os
import tempfile

import pytest
import torch

import plain_lilevik as P
from rbitnet_amd.cache import Cache
from rbitnet_amd.config.lilevik import LilevikConfig
from rbitnet_amd.config.spec import PartSpec
from rbitnet_amd.engine.context import StepBatch, StepContext
from rbitnet_amd.parts import BuildEnv, build_part
from rbitnet_amd.parts.stream import ExpertPairs, NormedTerm

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F64 = torch.float64
EPS = 1e-5
BOTH = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def _same_numbers_every_run():
    torch.manual_seed(20260117)


@pytest.fixture(scope="module")
def lib():
    from rbitnet_amd.csrc.lib import kernels
    return kernels()


def _env(lib, hidden, dtype):
    return BuildEnv(hidden_size=hidden, dtype=dtype, device=torch.device(DEV), lib=lib)


def _rel(got, want):
    want = want.double().cpu()
    return float((got.double().cpu() - want).abs().max() / want.abs().max().clamp_min(1e-30))


def _rms(got, want):
    want = want.double().cpu()
    return float(((got.double().cpu() - want) ** 2).mean().sqrt() / want.abs().max().clamp_min(1e-30))


def _close(got, want, dtype) -> bool:
    """float32: every value within 2e-5 of the largest.  bfloat16 rounds activations at every product's input: the root mean
    square error is bounded tightly (a wrong formula, chunk or state moves it by far more), the largest error loosely."""
    if dtype in (torch.float32, "float32"):
        return _rel(got, want) < 2e-5
    return _rms(got, want) < 1e-2 and _rel(got, want) < 1e-1


def _close_rows(got, want, dtype) -> bool:
    """Whole models.  bfloat16 is bounded row by row: a router's close call may go the other way for a token when its input is
    rounded, which moves that token's logits and little else, while a wrong mechanism moves every row it touches."""
    if dtype in (torch.float32, "float32"):
        return _rel(got, want) < 2e-5
    want = want.double().cpu()
    err = ((got.double().cpu() - want) ** 2).mean(-1).sqrt() / want.abs().max()
    return float(err.median()) < 2e-2 and float((err > 6e-2).double().mean()) <= 0.1


def _bf(t):
    return t.to(torch.bfloat16).to(F64)


def _step(lib, cache, slots, q_lens):
    past = [cache.length(s) for s in slots]
    cache.reserve(slots, q_lens)
    return StepContext.for_batch(DEV, StepBatch(slots, past, [[0] * q for q in q_lens], [], cache.block_tables(slots)),
                                 n_compute_units=lib.n_compute_units)


def _place(part, w, dtype):
    specs = part.tensor_specs()
    return {n: w[n].to(DEV, torch.float32 if specs[n].role == "gain" else dtype).contiguous() for n in specs}


def _requests(part):
    many = getattr(part, "cache_requests", None)
    return [many()] if many else [part.cache_request()]


def _run_mixer(lib, part, x, cuts, dtype, pages=8):
    """The mixer on x [T, E] fed in pieces of the given sizes, through a cache of its own."""
    cache = Cache(_requests(part), 2, 64 * pages, dtype, DEV)
    cache.alloc_slot()                                    # slot 0 stays idle: the sequence lives in slot 1
    slot = cache.alloc_slot()
    outs, at = [], 0
    for n in cuts:
        ctx = _step(lib, cache, [slot], [n])
        outs.append(part.forward(x[at:at + n].to(DEV, dtype).contiguous(), ctx, cache.view(0, ctx.block_tables)))
        cache.commit([slot], [n])
        at += n
    return torch.cat(outs)


def _mixer(lib, hidden, kind, m, dtype):
    cfg = LilevikConfig(vocab=4, width=hidden, norm_eps=EPS, layers=[{"type": kind, "mixer": m, "mlp": None}], max_positions=2048)
    cfg.check()
    return build_part("mixer", cfg.to_spec().layers[0].mixer, _env(lib, hidden, dtype))


def _mixer_weights(kind, hidden, m, seed):
    t = P.random_lilevik_tensors({"vocab": 4, "width": hidden, "layers": [{"type": kind, "mixer": m, "mlp": None}]}, seed)
    return {k[len("l0.mix."):]: v for k, v in t.items() if k.startswith("l0.mix.")}


CUTS = ([200], [63, 1, 1, 2, 61, 72], [130] + [1] * 70, [2] * 5 + [190])


# ---------------------------------------------------------------------------- the norm
@pytest.mark.parametrize("width,dtype", [(40, torch.float32), (256, torch.bfloat16), (51, torch.float32), (4100, torch.bfloat16), (33, torch.bfloat16)])
def test_the_tanh_norm_in_front_of_and_behind_a_sublayer(lib, width, dtype):
    tol = 2e-6 if dtype == torch.float32 else 6e-3

    def norm():
        part = build_part("norm", PartSpec("tanh", {"size": width, "names": {"weight": "", "bias": "b", "alpha": "alpha"}}), _env(lib, width, dtype))
        w = (torch.tensor(0.3 + 2 * float(torch.rand(())), dtype=F64), _bf(torch.randn(width, dtype=F64)), _bf(torch.randn(width, dtype=F64)))
        part.load({"alpha": w[0].float().to(DEV), "": w[1].float().to(DEV), "b": w[2].float().to(DEV)})
        return part, (w[0].float().double(), w[1], w[2])

    before, wb = norm()
    after, wa = norm()
    for n in (1, 9, 700):
        x = 3 * torch.randn(n, width, dtype=F64)
        x[0, :min(width, 8)] = torch.tensor([0.0, 1e-6, -1e-4, 40.0, -40.0, 1e-30, 0.5, -3.0], dtype=F64)[:min(width, 8)]
        x = x.float().double()
        dev = lambda t: t.float().to(DEV)
        assert _rel(before.forward(dev(x)), P.tanh_norm(x, *wb)) < tol
        y = torch.randn(n, width, dtype=F64)
        terms = torch.randn(5, n, width, dtype=F64)
        outputs, weights = torch.randn(n * 3, width, dtype=F64), torch.rand(n * 3, dtype=F64)
        total = (outputs * weights[:, None]).view(n, 3, width).sum(1)
        # (what is still to be added, the same in plain numbers)
        for delta, plain in ((dev(y), y), (dev(terms), terms.sum(0)), (NormedTerm(after, dev(y)), P.tanh_norm(y, *wa)),
                             (NormedTerm(after, dev(terms)), P.tanh_norm(terms.sum(0), *wa)),
                             (NormedTerm(after, ExpertPairs(dev(outputs), dev(weights))), P.tanh_norm(total, *wa))):
            xd = dev(x)
            h = before.forward(xd, delta)
            assert _rel(xd, x + plain) < 2e-6 and _rel(h, P.tanh_norm(x + plain, *wb)) < tol
            xd = dev(x)                                                   # chosen rows: the stream stays as it is
            rows = [n - 1, 0, n // 2]
            h = before.forward(xd, delta, torch.tensor(rows, dtype=torch.int32, device=DEV))
            assert torch.equal(xd, dev(x)) and _rel(h, P.tanh_norm(x + plain, *wb)[rows]) < tol
        xd = dev(x)
        after.add_normed(xd, ExpertPairs(dev(outputs), dev(weights)))
        assert _rel(xd, x + P.tanh_norm(total, *wa)) < 2e-6


def test_layers_with_norms_on_both_sides_take_other_norms_too(lib):
    """The block with RMS norms, which stand on an output but leave nothing to the norm that follows: x <- x + n1b(m(n1(x)))."""
    from rbitnet_amd.config.spec import LayerSpec
    from rbitnet_amd.parts.block import SandwichBlock
    e, t_len = 48, 70
    m = dict(heads=2, dim=8, vdim=8, decay=[0.9, 0.5])
    norm = lambda: PartSpec("rmsnorm", {"size": e, "eps": EPS})
    spec = LayerSpec(prefix="l", block="sandwich", mixer=PartSpec("lightning", dict(m, eps=EPS)), feed_forward=None, norm1=norm(), norm2=None,
                     params={"norm1b": norm()})
    block = SandwichBlock(spec, _env(lib, e, torch.float32))
    w = _mixer_weights("lightning", e, m, 3)
    g1, g2 = _bf(torch.randn(e, dtype=F64)), _bf(torch.randn(e, dtype=F64))
    block.norm1.load({"weight": g1.float().to(DEV)})
    block.norm1b.load({"weight": g2.float().to(DEV)})
    block.mixer.load(_place(block.mixer, w, torch.float32))
    x = torch.randn(t_len, e, dtype=F64)
    want = x + P.unit_rms(P.lightning(P.unit_rms(x, EPS) * g1, w, m, EPS), EPS) * g2
    cache = Cache([block.cache_requests()], 1, 128, torch.float32, DEV)
    slot = cache.alloc_slot()
    ctx = _step(lib, cache, [slot], [t_len])
    xd = x.float().to(DEV)
    assert block.forward(xd, None, ctx, cache.view(0, ctx.block_tables), next_norm=block.norm1) is None
    assert _rel(xd, want) < 2e-5


# ---------------------------------------------------------------------------- attention in chunks with sigmoid weights
def _att(heads, kv_heads, dim, vdim, dims, base, scale, chunk=None, scaling=None):
    out = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot={"base": base, "dims": dims})
    if scaling:
        out["rot"]["scaling"] = scaling
    if chunk:
        out["mask"] = {"size": chunk}
    return out


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}
ATTENTIONS = [
    _att(4, 2, 16, 24, 8, 100.0, 0.3, 36, YARN),
    _att(3, 3, 24, 8, 24, 5000.0, 0.2, 70),                       # all of the head rotated, chunks across page borders
    _att(8, 2, 64, 64, 32, 1e4, 0.12, 64, YARN),                  # the matrix cores' sizes, a chunk a page
    _att(6, 3, 64, 128, 16, 5e5, 0.1, 129),                       # values larger than keys
    _att(6, 1, 100, 36, 20, 1e4, 0.1, 100, YARN),                 # padded to 128 for the matrix cores
    _att(1, 1, 6, 5, 0, 10.0, 1.0, 1),                            # a chunk of one, one head, no rotation
    _att(2, 1, 128, 64, 128, 300.0, 0.08),                        # no chunks
    _att(5, 5, 7, 9, 6, 20.0, 0.4, 3),                            # odd sizes
    _att(34, 2, 32, 32, 16, 50.0, 0.15, 90),                      # 17 heads on a key head
    _att(2, 2, 160, 192, 2, 1e3, 0.06, 50),                       # beyond the matrix cores' sizes
    _att(4, 4, 12, 10, 6, 1e3, 0.3, 65, YARN),                    # a rotated part that is no multiple of 4
]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("p", ATTENTIONS)
def test_attention_whole_in_pieces_and_token_by_token(lib, p, dtype):
    hidden = 64
    part = _mixer(lib, hidden, "attention", p, dtype)
    w = _mixer_weights("attention", hidden, p, seed=p["heads"] + p["dim"])
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(200, hidden, dtype=F64))
    want = P.attention(x, w, p, EPS)
    for cuts in CUTS:
        assert _close(_run_mixer(lib, part, x, cuts, dtype), want, dtype), cuts


def test_what_the_cache_holds_are_normed_rotated_keys_and_normed_values(lib):
    hidden, t_len = 64, 70
    for dtype in BOTH:
        for p in (ATTENTIONS[0], ATTENTIONS[4], ATTENTIONS[7], ATTENTIONS[10]):
            part = _mixer(lib, hidden, "attention", p, dtype)
            w = _mixer_weights("attention", hidden, p, seed=1)
            part.load(_place(part, w, dtype))
            x = _bf(torch.randn(t_len, hidden, dtype=F64))
            cache = Cache([part.cache_requests()], 1, 256, dtype, DEV)
            slot = cache.alloc_slot()
            ctx = _step(lib, cache, [slot], [t_len])
            view = cache.view(0, ctx.block_tables)
            part.forward(x.to(DEV, dtype), ctx, view)
            _, k, v = P.prepared_heads(x, w, p, EPS)
            pages = view.block_table[0].tolist()
            for t in (0, 1, 63, 64, t_len - 1):
                row_k, row_v = view.k_pages[pages[t // 64], :, t % 64], view.v_pages[pages[t // 64], :, t % 64]
                tol = 1e-5 if dtype == torch.float32 else 1e-2
                assert _rel(row_k[:, :p["dim"]], k[t]) < tol and _rel(row_v[:, :p["vdim"]], v[t]) < tol
                assert float(row_k[:, p["dim"]:].float().abs().sum()) == 0.0 and float(row_v[:, p["vdim"]:].float().abs().sum()) == 0.0


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("chunk,dim,vdim", [(36, 16, 12), (64, 64, 64), (65, 64, 128), (7, 8, 12), (130, 128, 48)])
def test_a_key_that_stands_out_at_every_edge_of_a_chunk(lib, dtype, chunk, dim, vdim):
    """One earlier token has the query's own input, keys are made from the matrix that makes queries, and the number added to
    the scores is so low that hardly any other key has a weight: seen as the first and the last but one of the query's chunk,
    and not as the last of the chunk before; in a prompt and in decoding, with the query at the chunk's end and at its start."""
    hidden = 64
    p = _att(2, 1, dim, vdim, 2, 1e9, 24.0 / dim, chunk)                # the rotated pair hardly turns
    w = _mixer_weights("attention", hidden, p, seed=chunk)
    w["k"] = w["q"][:dim].clone()
    w["q"] = torch.cat([w["k"], w["k"]])                                # both heads alike: the whole norm is then each head's own
    w["q.norm"], w["k.norm"] = torch.ones(2 * dim, dtype=F64), torch.ones(dim, dtype=F64)
    w["pb"] = torch.full((2,), -14.0, dtype=F64)
    part = _mixer(lib, hidden, "attention", p, dtype)
    part.load(_place(part, w, dtype))
    for n in (1, 3):
        start = n * chunk
        t_len = start + chunk + 3
        end = start + chunk - 1
        for query, at, seen in ((end, start, True), (end, start - 1, False), (start, start - 1, False), (end, end - 1, True),
                                (start + chunk // 2, start, True), (start + chunk, end, False)):
            if at == query:
                continue
            x = _bf(torch.randn(t_len, hidden, dtype=F64))
            x[at] = x[query]
            q, k, _ = P.prepared_heads(x, w, p, EPS)
            a = P.sigmoid_weights(q, k, p["scale"], w["pb"], P.visible(t_len, chunk))
            if seen:
                assert float(a[0, query, at]) > 0.5                     # the edge shows in the plain weights
            else:
                assert float(a[:, query, at].max()) == 0.0
            want = P.attention(x, w, p, EPS)
            for cuts in ([t_len], [query] + [1] * (t_len - query), [at + 1, t_len - at - 1]):
                got = _run_mixer(lib, part, x, cuts, dtype, pages=10)
                assert _close(got, want, dtype), (query, at, cuts)
                assert _close(got[query], want[query], dtype), (query, at, cuts)


@pytest.mark.parametrize("dtype", BOTH)
def test_a_far_key_among_hundreds(lib, dtype):
    """Token 2 has the input of a query 620 tokens later, at whose distance the (stretched, scaled) rotation must be turned by
    the true positions; every other key's weight is next to nothing."""
    hidden, t_len, dim = 64, 640, 64
    p = _att(4, 2, dim, 64, 32, 1e4, 0.4, None, {"factor": 8.0, "original": 256, "fast": 4.0, "slow": 0.5})
    w = _mixer_weights("attention", hidden, p, seed=5)
    w["k"] = torch.cat([w["q"][:dim], w["q"][2 * dim:3 * dim]])
    w["pb"] = torch.full((4,), -9.0, dtype=F64)
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    x[2] = x[622]
    want = P.attention(x, w, p, EPS)
    other = x.clone()
    other[2] = _bf(torch.randn(hidden, dtype=F64))
    assert _rel(want[622], P.attention(other, w, p, EPS)[622]) > 0.05      # the far token matters to its query
    part = _mixer(lib, hidden, "attention", p, dtype)
    part.load(_place(part, w, dtype))
    for cuts in ([t_len], [600] + [1] * 40, [2, 400, 238]):
        got = _run_mixer(lib, part, x, cuts, dtype, pages=11)
        assert _close(got, want, dtype) and _close(got[622], want[622], dtype), cuts


@pytest.mark.parametrize("splits", [1, 3, 16])
@pytest.mark.parametrize("chunk", [None, 500])
def test_long_decoding_with_the_pages_dealt_to_several_workgroups(lib, chunk, splits):
    """1,100 tokens, the last 60 one by one, across a chunk's border; the number of shares forced, as a long context would
    choose it."""
    from rbitnet_amd.engine import context as C
    hidden, t_len = 64, 1100
    p = _att(8, 2, 64, 64, 32, 1e4, 0.125, chunk)
    w = _mixer_weights("attention", hidden, p, seed=11)
    w["pb"] = w["pb"] - 3.0
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    want = P.attention(x, w, p, EPS)
    part = _mixer(lib, hidden, "attention", p, torch.bfloat16)
    part.load(_place(part, w, torch.bfloat16))
    first = (1000 if chunk else t_len) - 30
    C.FORCED_DECODE_SPLITS = splits
    try:
        got = _run_mixer(lib, part, x, [first] + [1] * 60 + ([t_len - first - 60] if t_len > first + 60 else []), torch.bfloat16, pages=20) \
            if chunk else _run_mixer(lib, part, x, [t_len - 60] + [1] * 60, torch.bfloat16, pages=20)
    finally:
        C.FORCED_DECODE_SPLITS = None
    assert _close(got, want, torch.bfloat16)
    assert _close(got[first - 30:first + 30], want[first - 30:first + 30], torch.bfloat16)


def test_attention_of_several_sequences_that_go_on_at_unequal_lengths(lib):
    """Three sequences in one step, on top of unequal pasts, against each alone; slots and pages are then freed and used
    again by other sequences."""
    hidden, p = 64, _att(8, 2, 64, 64, 32, 1e4, 0.12, 100, YARN)
    w = _mixer_weights("attention", hidden, p, seed=4)
    for dtype in BOTH:
        part = _mixer(lib, hidden, "attention", p, dtype)
        part.load(_place(part, w, dtype))
        cache = Cache([part.cache_requests()], 4, 64 * 14, dtype, DEV)
        for lens in ((150, 3, 230), (99, 201, 64)):
            xs = [_bf(torch.randn(n, hidden, dtype=F64)) for n in lens]
            slots = [cache.alloc_slot() for _ in xs]
            at, outs = [0, 0, 0], [[], [], []]
            while any(a < n for a, n in zip(at, lens)):
                live = [i for i in range(3) if at[i] < lens[i]]
                take = [min(lens[i] - at[i], 1 + 60 * (i + 1)) for i in live]
                ctx = _step(lib, cache, [slots[i] for i in live], take)
                y = part.forward(torch.cat([xs[i][at[i]:at[i] + n] for i, n in zip(live, take)]).to(DEV, dtype), ctx, cache.view(0, ctx.block_tables))
                off = 0
                for i, n in zip(live, take):
                    outs[i].append(y[off:off + n])
                    off += n
                    at[i] += n
                cache.commit([slots[i] for i in live], take)
            for i in range(3):
                assert _close(torch.cat(outs[i]), P.attention(xs[i], w, p, EPS), dtype), (lens, i)
            for s in slots:
                cache.free_slot(s)
            cache.check()


# ---------------------------------------------------------------------------- attention through a latent
def _lat(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base):
    out = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale)
    if rot_dim:
        out["rot"] = {"base": base, "dims": rot_dim}
    return out


LATENTS = [_lat(3, 8, 4, 6, 12, 10, 0.3, 100.0), _lat(4, 32, 32, 16, 48, 96, 0.1, 1e4), _lat(16, 16, 16, 24, 32, 40, 0.15, 5e5),
           _lat(1, 5, 2, 7, 3, 9, 0.5, 7.0), _lat(20, 24, 8, 8, 64, 64, 0.12, 300.0), _lat(2, 64, 64, 64, 128, 192, 0.08, 1e4),
           _lat(5, 48, 16, 72, 40, 112, 0.1, 1e4), _lat(4, 16, 0, 16, 24, 64, 0.2, 1.0), _lat(6, 64, 64, 128, 96, 64, 0.09, 1e5)]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("p", LATENTS)
def test_latent_attention_whole_in_pieces_and_token_by_token(lib, p, dtype):
    hidden = 64
    part = _mixer(lib, hidden, "latent_attention", p, dtype)
    w = _mixer_weights("latent_attention", hidden, p, seed=p["heads"] + p["dim"])
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(200, hidden, dtype=F64))
    want = P.latent_attention(x, w, p, EPS)
    for cuts in CUTS:
        assert _close(_run_mixer(lib, part, x, cuts, dtype), want, dtype), cuts


@pytest.mark.parametrize("dtype", BOTH)
def test_a_far_token_through_the_latent(lib, dtype):
    hidden, t_len = 64, 640
    p = _lat(4, 32, 32, 32, 64, 96, 0.18, 1e4)
    w = _mixer_weights("latent_attention", hidden, p, seed=9)
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    x[2] = x[2] * 4
    want = P.latent_attention(x, w, p, EPS)
    base = P.latent_attention(torch.cat([x[:2], x[3:]]), w, p, EPS)
    assert _rel(want[630:], base[629:]) > 1e-2                                  # the far token matters to the last ones
    part = _mixer(lib, hidden, "latent_attention", p, dtype)
    part.load(_place(part, w, dtype))
    for cuts in ([t_len], [600] + [1] * 40):
        assert _close(_run_mixer(lib, part, x, cuts, dtype, pages=11), want, dtype), cuts


# ---------------------------------------------------------------------------- lightning attention
LIGHTNINGS = [dict(heads=2, dim=32, vdim=48, decay=[0.55, 0.998]), dict(heads=3, dim=12, vdim=20, decay=[0.0, 1.0, 0.9]),
              dict(heads=1, dim=64, vdim=64, decay=[0.97]), dict(heads=6, dim=5, vdim=7, decay=[0.5, 0.6, 0.7, 0.8, 0.9, 0.99]),
              dict(heads=2, dim=128, vdim=24, decay=[0.95, 0.3]), dict(heads=2, dim=20, vdim=128, decay=[0.999, 0.9999]),
              dict(heads=2, dim=100, vdim=100, decay=[0.99, -0.5]), dict(heads=1, dim=160, vdim=16, decay=[0.9]),
              dict(heads=3, dim=1, vdim=1, decay=[0.9, 0.8, 0.99]), dict(heads=2, dim=16, vdim=200, decay=[0.9, 0.99])]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("p", LIGHTNINGS)
def test_lightning_attention_whole_in_pieces_and_token_by_token(lib, p, dtype):
    hidden = 48
    part = _mixer(lib, hidden, "lightning", p, dtype)
    w = _mixer_weights("lightning", hidden, p, seed=p["heads"] + p["dim"])
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(200, hidden, dtype=F64))
    want = P.lightning(x, w, p, EPS)
    for cuts in CUTS + ([64, 64, 64, 8], [65, 127, 8], [1] * 20 + [180]):
        assert _close(_run_mixer(lib, part, x, cuts, dtype), want, dtype), cuts


@pytest.mark.parametrize("dim,vdim", [(64, 64), (128, 128), (64, 112), (92, 20)])
def test_chunks_on_the_matrix_cores_against_the_plain_sum(lib, dim, vdim):
    """The kernel alone, float32: three sequences on top of states that are not zero, piece lengths at and around a chunk."""
    heads, decay = 3, [0.9, 0.999, 1.0]
    for lens in ((64, 1, 130), (63, 65, 2), (128, 200, 5)):
        t = sum(lens)
        qkv = torch.randn(t, heads * (2 * dim + vdim), dtype=F64)
        state = torch.randn(5, heads, vdim, dim, dtype=F64)
        slots = [4, 0, 2]
        powers = torch.stack([torch.tensor(decay, dtype=F64) ** i for i in range(65)], 1).float().to(DEV).contiguous()

        class Ctx:
            n_tokens, n_seqs = t, 3
            cu_seqlens = torch.tensor([0, lens[0], lens[0] + lens[1], t], dtype=torch.int32, device=DEV)
        Ctx.slots = torch.tensor(slots, dtype=torch.int32, device=DEV)
        sd, out = state.float().to(DEV), torch.empty(t, heads * vdim, device=DEV)
        lib.lightning_chunks(qkv.float().to(DEV), dim, heads, vdim, powers, sd, Ctx, out)
        q, k, v = (P.silu(a) for a in qkv.split([heads * dim, heads * dim, heads * vdim], 1))
        at = 0
        for n, slot in zip(lens, slots):
            qq, kk, vv = (a[at:at + n].view(n, heads, -1) for a in (q, k, v))
            s0 = state[slot].transpose(1, 2)                       # [head, key channel, value channel]
            d = torch.tensor(decay, dtype=F64)
            want = P.decaying_sum(qq, kk, vv, d)
            i = torch.arange(1, n + 1, dtype=F64)
            want = want + torch.einsum("th,hkv,thk->thv", d[None, :] ** i[:, None], s0, qq)
            assert _rel(out[at:at + n], want.reshape(n, -1)) < 2e-5, (lens, slot)
            end = s0 * d[:, None, None] ** n + sum(d[:, None, None] ** (n - 1 - j) * kk[j][:, :, None] * vv[j][:, None, :] for j in range(n))
            assert _rel(sd[slot].transpose(1, 2), end) < 2e-5
            at += n
        for slot in (1, 3):                                         # nobody's slots stay as they were
            assert torch.equal(sd[slot].cpu(), state[slot].float())


def test_what_the_first_token_wrote_is_read_much_later_beside_another_sequence(lib):
    """Decays of nearly 1: the state keeps the first token's k v^T for 260 tokens; a second sequence in another slot, fed in
    the same steps, keeps its own; a slot that is freed and handed out again starts at zero."""
    hidden, p, t_len = 32, dict(heads=2, dim=16, vdim=16, decay=[1.0, 0.9999]), 260
    part = _mixer(lib, hidden, "lightning", p, torch.float32)
    w = _mixer_weights("lightning", hidden, p, seed=3)
    part.load(_place(part, w, torch.float32))
    cache = Cache(_requests(part), 3, 64, torch.float32, DEV)
    cache.alloc_slot()
    for _ in range(2):
        xs = [_bf(torch.randn(t_len, hidden, dtype=F64)) for _ in range(2)]
        xs[0][0] = xs[0][0] * 6
        wants = [P.lightning(x, w, p, EPS) for x in xs]
        gone = P.lightning(torch.cat([torch.zeros(1, hidden, dtype=F64), xs[0][1:]]), w, p, EPS)
        assert _rel(wants[0][-1:], gone[-1:]) > 1e-2                                # the first token still matters at the end
        slots = [cache.alloc_slot(), cache.alloc_slot()]
        outs, at = [[], []], 0
        for n in [100, 1, 1, 2, 156]:
            ctx = _step(lib, cache, slots, [n, n])
            x = torch.cat([xs[0][at:at + n], xs[1][at:at + n]]).to(DEV, torch.float32)
            y = part.forward(x, ctx, cache.view(0, ctx.block_tables))
            outs[0].append(y[:n])
            outs[1].append(y[n:])
            cache.commit(slots, [n, n])
            at += n
        for i in range(2):
            assert _close(torch.cat(outs[i]), wants[i], torch.float32), i
        for s in slots:
            cache.free_slot(s)


# ---------------------------------------------------------------------------- routed experts
EXPERTS = [(64, 32, 4, 2, 70), (48, 24, 7, 3, 33), (32, 16, 1, 1, 9), (128, 64, 16, 4, 300), (50, 31, 5, 5, 20), (64, 96, 130, 6, 40),
           (224, 96, 11, 3, 1), (96, 64, 9, 2, 32), (64, 32, 70, 64, 5)]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("hidden,ff,experts,top,t_len", EXPERTS)
def test_experts_by_the_softmax_over_the_chosen(lib, dtype, hidden, ff, experts, top, t_len):
    spec = PartSpec("routed_experts", {"experts": experts, "top": top, "intermediate_size": ff, "limit": None, "score": "chosen", "bias": True,
                                       "weight_on": "output"})
    part = build_part("feed_forward", spec, _env(lib, hidden, dtype))
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    t = P.random_lilevik_tensors({"vocab": 4, "width": hidden, "layers": [{"type": "lightning", "mixer": dict(heads=1, dim=4, vdim=4, decay=[1.0]),
                                                                           "mlp": mlp}]}, seed=experts + top)
    w = {k[len("l0.mlp."):]: v for k, v in t.items() if k.startswith("l0.mlp.")}
    # a bias that takes half of the experts out of the choice, and makes the others' logits large as numbers
    if 2 * top <= experts:
        w["router.b"] = torch.where(torch.arange(experts) % 2 == 0, 24.0, 0.0).to(F64) + w["router.b"]
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    want = P.experts(x, w, mlp)
    total = part.forward(x.to(DEV, dtype))
    pairs = part.forward(x.to(DEV, dtype), pairs=True)
    summed = (pairs.outputs.view(t_len, top, hidden) * pairs.weights.view(t_len, top, 1)).sum(1)
    assert _close(total, want, dtype) and _close(summed, want, dtype)
    assert torch.allclose(pairs.weights.view(t_len, top).sum(1), torch.ones(t_len, device=DEV), atol=1e-5)
    alone = torch.cat([part.forward(x[i:i + 1].to(DEV, dtype)) for i in range(min(t_len, 6))])      # the same whatever else a step holds
    assert _rel(alone, total[:len(alone)].double().cpu()) < 1e-5
    for n in (2, 16, 17, 48, 64, 65):                            # the kernels for few tokens and those for many add up alike
        if n < t_len:
            assert _rel(part.forward(x[:n].to(DEV, dtype)), total[:n].double().cpu()) < 1e-5, n


# ---------------------------------------------------------------------------- whole models
def _moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def _lig(heads, dim, vdim, *decay):
    return dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay))


# everything different from layer to layer
MODEL_A = {"architecture": "Lilevik", "vocab": 96, "width": 64, "norm": {"eps": 1e-5}, "layers": [
    {"type": "lightning", "mixer": _lig(3, 12, 20, 0.5, 0.9, 0.995), "mlp": _moe(24, 5, 2)},
    {"type": "attention", "mixer": _att(4, 2, 16, 24, 8, 100.0, 0.3, 44, YARN), "mlp": None},
    {"type": "latent_attention", "mixer": _lat(3, 8, 4, 6, 12, 10, 0.3, 100.0), "mlp": _moe(40, 3, 3)},
    {"type": "attention", "mixer": _att(3, 3, 24, 8, 24, 5e3, 0.2, 9), "mlp": _moe(16, 8, 1)},
    {"type": "lightning", "mixer": _lig(2, 32, 8, 0.99, 0.7), "mlp": None},
    {"type": "latent_attention", "mixer": _lat(4, 16, 8, 12, 24, 40, 0.2, 5e4), "mlp": _moe(32, 6, 4)}]}
# values that a model may happen to make equal or 1
MODEL_B = {"architecture": "Lilevik", "vocab": 50, "width": 32, "norm": {"eps": 1e-6}, "layers": [
    {"type": "attention", "mixer": _att(1, 1, 32, 32, 32, 1e4, 1.0, 1), "mlp": _moe(32, 1, 1)},
    {"type": "lightning", "mixer": _lig(1, 32, 32, 1.0), "mlp": _moe(32, 2, 2)},
    {"type": "latent_attention", "mixer": _lat(1, 32, 32, 32, 32, 32, 1.0, 1e4), "mlp": None}]}
# sizes on the matrix cores' grid
MODEL_C = {"architecture": "Lilevik", "vocab": 320, "width": 128, "norm": {"eps": 1e-5}, "layers": [
    {"type": "attention", "mixer": _att(8, 2, 64, 64, 32, 2e5, 0.12, 128, {"factor": 6.0, "original": 256, "fast": 16.0, "slow": 1.0}), "mlp": _moe(64, 6, 2)},
    {"type": "lightning", "mixer": _lig(2, 64, 64, 0.95, 0.999), "mlp": _moe(128, 4, 2)},
    {"type": "latent_attention", "mixer": _lat(8, 32, 32, 32, 64, 96, 0.12, 1e4), "mlp": _moe(64, 8, 3)},
    {"type": "attention", "mixer": _att(4, 4, 128, 64, 64, 1e4, 0.09, 70), "mlp": _moe(64, 4, 1)}]}
# sizes off every grid
MODEL_D = {"architecture": "Lilevik", "vocab": 37, "width": 50, "norm": {"eps": 1e-4}, "layers": [
    {"type": "latent_attention", "mixer": _lat(5, 6, 2, 7, 9, 11, 0.4, 7.0), "mlp": _moe(31, 3, 2)},
    {"type": "attention", "mixer": _att(3, 1, 10, 14, 6, 33.0, 0.3, 3), "mlp": _moe(9, 4, 2)},
    {"type": "lightning", "mixer": _lig(3, 5, 3, 0.9, 0.99, 0.2), "mlp": None},
    {"type": "attention", "mixer": _att(5, 5, 6, 6, 2, 7.0, 0.4, 67, {"factor": 3.0, "original": 16, "fast": 2.0, "slow": 0.5}), "mlp": _moe(7, 5, 1)}]}
MODELS = {"A": (MODEL_A, 21), "B": (MODEL_B, 22), "C": (MODEL_C, 23), "D": (MODEL_D, 24)}
_TMP = tempfile.TemporaryDirectory(prefix="lilevik_models_")
_MADE = {}


def _write(folder, cfg, tensors):
    from rbitnet_amd.weights.safetensors_io import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(os.path.join(folder, "model.safetensors"), [(k, v.to(torch.bfloat16)) for k, v in tensors.items()])


def _model(name):
    """(folder, oracle) of a model written once per session."""
    if name not in _MADE:
        cfg, seed = MODELS[name]
        tensors = P.random_lilevik_tensors(cfg, seed)
        folder = os.path.join(_TMP.name, name)
        _write(folder, cfg, tensors)
        _MADE[name] = (folder, P.PlainLilevik(copy.deepcopy(cfg), tensors))
    return _MADE[name]


def _tokens(name, n, seed):
    g = torch.Generator().manual_seed(100 * seed + n)
    return torch.randint(0, MODELS[name][0]["vocab"], (n,), generator=g).tolist()


def _engine(name, dtype, **kw):
    import rbitnet_amd
    return rbitnet_amd.Engine.load_path(_model(name)[0], dtype=dtype, max_seq_len=1024, **kw)


@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_every_layer_of_a_model_against_the_plain_stream(name):
    """The residual stream after every layer (float32), so that a fault names its layer."""
    from rbitnet_amd.parts import block as B
    eng = _engine(name, "float32", max_tokens=64 * 4, max_batch=1)
    toks = _tokens(name, 90, 4)
    want = _model(name)[1].streams(toks)[1:]
    seen = []
    orig = B.SandwichBlock.forward

    def traced(self, x, pending, ctx, view, next_norm=None):
        out = orig(self, x, pending, ctx, view, next_norm)
        whole = x.detach().clone()
        if out is not None:
            out.apply(whole)                       # what the next norm still has to add
        seen.append(whole.cpu())
        return out

    B.SandwichBlock.forward = traced
    try:
        slot = eng.alloc_slot()
        eng.use_plans = False
        eng.step([(slot, toks)], "last")
    finally:
        B.SandwichBlock.forward = orig
    assert len(seen) == len(want)
    for i, (g, w) in enumerate(zip(seen, want)):
        assert _rel(g, w) < 2e-5, i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_model_whole_in_pieces_and_decoded(name, dtype):
    eng = _engine(name, dtype, max_tokens=64 * 12, max_batch=3)
    toks = _tokens(name, 200, 1)
    want = _model(name)[1].logits(toks)
    for cuts in ([200], [130] + [1] * 70, [2, 2, 3, 57, 64, 1, 65, 6], [1] * 5 + [195]):
        slot = eng.alloc_slot()
        out, at = [], 0
        for n in cuts:
            out.append(eng.step([(slot, toks[at:at + n])], "all"))
            at += n
        eng.free_slot(slot)
        assert _close_rows(torch.cat(out), want, dtype), cuts


def _together(eng, seqs, heads, leave):
    """The requests start together, then go on token by token; request i leaves after leave[i] tokens.  -> logits of each"""
    slots = [eng.alloc_slot() for _ in seqs]
    logits = eng.step([(sl, s[:n]) for sl, s, n in zip(slots, seqs, heads)], "all")
    got, off = [], 0
    for n in heads:
        got.append([logits[off:off + n]])
        off += n
    at, live = list(heads), [i for i in range(len(seqs)) if heads[i] < leave[i]]
    for i in set(range(len(seqs))) - set(live):
        eng.free_slot(slots[i])
    while live:
        logits = eng.step([(slots[i], [seqs[i][at[i]]]) for i in live], "last")
        for row, i in enumerate(live):
            got[i].append(logits[row:row + 1])
            at[i] += 1
        for i in [i for i in live if at[i] >= leave[i]]:
            eng.free_slot(slots[i])
            live.remove(i)
    eng.cache.check()
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_batches_of_unequal_requests_and_slots_used_again(name, dtype):
    """Four requests of 1 to 150 tokens start together and are decoded together, the short ones leaving early; then two
    new requests take the freed slots and pages.  Every request's logits are those it has alone."""
    eng = _engine(name, dtype, max_tokens=64 * 8, max_batch=4)
    oracle = _model(name)[1]
    for wave, lens in enumerate(([1, 150, 67, 30], [64, 129])):
        seqs = [_tokens(name, n + 12, 7 + wave) for n in lens]
        leave = [n + (3 + 4 * i if i < 3 else 12) for i, n in enumerate(lens)]
        got = _together(eng, seqs, lens, leave)
        for i, g in enumerate(got):
            assert g.shape[0] == leave[i]
            assert _close_rows(g, oracle.logits(seqs[i])[:leave[i]], dtype), (wave, i)


@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("C", "bfloat16"), ("C", "float32")])
def test_long_decoding_and_greedy_generation_through_the_engine(name, dtype):
    """Greedy generation through `Engine.generate` (its scheduler, its captured decode step) gives the plain
    implementation's greedy tokens for a batch of unequal prompts, past chunks of every layer."""
    eng = _engine(name, dtype, max_tokens=64 * 16, max_batch=5)
    oracle = _model(name)[1]
    limits = (150, 40, 90, 12, 25)
    prompts = [_tokens(name, n, 3) for n in (5, 70, 1, 33, 64)]
    results = eng.generate(prompts, max_tokens=list(limits), temperature=0.0)
    for p, r, n in zip(prompts, results, limits):
        assert len(r.tokens) == n and r.finish_reason == "length"
        seq = list(p) + r.tokens
        logits = oracle.logits(seq[:-1])[len(p) - 1:]
        top2 = logits.topk(2, dim=-1)
        margin = (1e-4 if dtype == "float32" else 0.08) * float(logits.abs().max())
        clear = (top2.values[:, 0] - top2.values[:, 1]) > margin          # a tie within rounding may go either way
        same = sum(1 for g, t, c in zip(top2.indices[:, 0].tolist(), r.tokens, clear.tolist()) if c and g == t)
        assert same >= (1.0 if dtype == "float32" else 0.95) * int(clear.sum())
        assert int(clear.sum()) > (0.9 if dtype == "float32" else 0.4) * n
    assert eng.stats["decode_tokens"] > 0 and eng.model.graph_safe and eng.model.plan_safe


def _random_config(rng):
    """A model whose every size, constant and layer order is drawn: what no hand-made model thought of."""
    def rotation(limit, zero=True):
        dims = rng.choice([d for d in ([0] if zero else []) + [2, 6, 8, 16, 32, 64, limit - limit % 2] if d <= limit])
        out = {"base": rng.choice([100.0, 1e4, 5e5]), "dims": dims}
        if dims and rng.random() < 0.6:
            out["scaling"] = {"factor": rng.choice([1.5, 4.0, 16.0]), "original": rng.choice([16, 128, 4096]), "fast": rng.choice([4.0, 32.0]),
                              "slow": rng.choice([0.5, 1.0])}
        return out

    def mixer(kind):
        if kind == "lightning":
            h = rng.choice([1, 2, 3, 4, 6])
            return dict(heads=h, dim=rng.choice([8, 12, 16, 32, 64, 96, 128]), vdim=rng.choice([8, 16, 20, 32, 64, 128]),
                        decay=[rng.choice([0.3, 0.62, 0.9, 0.98, 0.9995]) for _ in range(h)])
        if kind == "attention":
            dim, kvh, group = rng.choice([8, 16, 32, 48, 64, 96, 128]), rng.choice([1, 2, 3, 4]), rng.choice([1, 2, 3, 4, 8, 20])
            out = dict(heads=kvh * group, kv_heads=kvh, dim=dim, vdim=rng.choice([8, 16, 32, 48, 64, 128]), scale=rng.choice([0.05, 0.125, 0.3]), rot=rotation(dim))
            if rng.random() < 0.9:
                out["mask"] = {"size": rng.choice([1, 7, 16, 36, 64, 65, 100, 128, 200])}
            return out
        rot = rng.choice([0, 2, 4, 8, 16, 32, 64])
        out = _lat(rng.choice([1, 2, 3, 4, 8, 16, 24, 32]), rng.choice([8, 16, 32, 64, 128]), rot, rng.choice([8, 16, 32, 64, 72]),
                   rng.choice([16, 24, 64, 88, 128]), rng.choice([8, 24, 32, 48, 64, 96, 112, 128]), rng.choice([0.05, 0.125, 0.2]), rng.choice([100.0, 1e4, 5e5]))
        return out

    layers = []
    for _ in range(rng.choice([2, 3, 4, 5])):
        kind = rng.choice(["latent_attention", "attention", "lightning"])
        n = rng.choice([1, 2, 5, 8, 12, 20])
        mlp = None if rng.random() < 0.2 else _moe(rng.choice([8, 16, 40, 64, 96]), n, rng.randint(1, min(n, 4)))
        layers.append({"type": kind, "mixer": mixer(kind), "mlp": mlp})
    return {"architecture": "Lilevik", "vocab": rng.choice([37, 96, 300, 512]), "width": rng.choice([32, 48, 64, 96, 128, 160, 256, 320]),
            "norm": {"eps": rng.choice([1e-5, 1e-6])}, "layers": layers}


@pytest.mark.parametrize("seed", list(range(40, 52)))
def test_models_drawn_at_random_whole_in_pieces_decoded_and_batched(seed, tmp_path):
    import random
    import rbitnet_amd
    cfg = _random_config(random.Random(seed))
    tensors = P.random_lilevik_tensors(cfg, seed)
    oracle = P.PlainLilevik(copy.deepcopy(cfg), tensors)
    _write(str(tmp_path), cfg, tensors)
    g = torch.Generator().manual_seed(seed)
    seqs = [torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for n in (210, 75, 9)]
    want = [oracle.logits(s) for s in seqs]
    for dtype in ("float32", "bfloat16"):
        eng = rbitnet_amd.Engine.load_path(str(tmp_path), dtype=dtype, max_seq_len=512, max_tokens=64 * 12, max_batch=4)
        slot = eng.alloc_slot()
        runs = [(eng.step([(slot, seqs[0])], "all"), want[0])]
        eng.free_slot(slot)
        slot, parts, at = eng.alloc_slot(), [], 0
        for n in [3, 61, 2, 64, 40] + [1] * 40:
            parts.append(eng.step([(slot, seqs[0][at:at + n])], "all"))
            at += n
        eng.free_slot(slot)
        runs.append((torch.cat(parts), want[0]))
        runs += list(zip(_together(eng, seqs, [180, 60, 1], [len(s) for s in seqs]), want))
        for i, (got, ref) in enumerate(runs):
            err = ((got.double().cpu() - ref) ** 2).mean(-1).sqrt() / ref.abs().max()
            if dtype == "float32":
                assert float(err.max()) < 5e-5, (seed, i)
            else:
                assert float(err.median()) < 2.5e-2 and float((err > 8e-2).double().mean()) <= 0.12, (seed, i)
        del eng


def test_replay_and_command_line_on_a_model_of_this_design(tmp_path, capsys):
    import numpy as np
    from rbitnet_amd import cli
    from rbitnet_amd.replay import replay
    folder, oracle = _model("D")
    eng = _engine("D", "float32", max_tokens=64 * 6, max_batch=4)
    a, b = _tokens("D", 70, 5), _tokens("D", 9, 6)
    lines = [json.dumps({"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [0, 65]},
                                                {"id": "b", "tokens": b[:8], "want": []}], "end": []}),
             json.dumps({"step": 1, "entries": [{"id": "a", "tokens": a[66:67], "want": [0]},
                                                {"id": "b", "tokens": b[8:9], "want": [0]}], "end": ["b"]}),
             json.dumps({"step": 2, "entries": [{"id": "a", "tokens": a[67:], "want": [2]}], "end": ["a"]})]
    log = io.StringIO()
    assert replay(eng, io.StringIO("\n".join(lines) + "\n"), str(tmp_path / "out"), log=log) == 3
    wa, wb = oracle.logits(a), oracle.logits(b)
    vocab = MODELS["D"][0]["vocab"]
    got = [np.fromfile(tmp_path / "out" / f"{i}.f32", dtype="<f4").reshape(-1, vocab) for i in range(3)]
    assert _close(torch.from_numpy(got[0]), wa[[0, 65]], "float32")
    assert _close(torch.from_numpy(got[1]), torch.stack([wa[66], wb[8]]), "float32")
    assert _close(torch.from_numpy(got[2]), wa[[69]], "float32")
    assert eng.cache.live_slots == []
    del eng
    capsys.readouterr()
    assert cli.main(["generate", "--model", folder, "--dtype", "float32", "--prompt-ids", ",".join(str(t) for t in b),
                     "--max-tokens", "5", "--temperature", "0"]) == 0
    rec = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert len(rec["tokens"]) == 5 and rec["tokens"][0] == int(oracle.logits(b)[-1].argmax())
