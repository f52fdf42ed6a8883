"""The Goperax parts and whole models on the GPU against the plain implementation of `plain_goperax.py`: each mechanism alone; a
prompt whole, in pieces down to two tokens and token by token; batches of unequal requests against each alone; slots, pages
and states used again; keys far away, at page borders, just inside and just outside every window, in prompts and in decoding;
the first tokens of a sequence; long decoding; sizes that differ in everything (and values that a model may happen to make equal
or 1); greedy generation through `Engine.generate`.  Configurations and weights are made here."""
import copy
import io
import json
import os
import tempfile

import pytest
import torch

import plain_goperax as P
from rbitnet_amd.cache import Cache
from rbitnet_amd.config.goperax import GoperaxConfig
from rbitnet_amd.config.spec import PartSpec
from rbitnet_amd.engine.context import StepBatch, StepContext
from rbitnet_amd.parts import BuildEnv, build_part
from rbitnet_amd.parts.stream import ExpertPairs, StreamsUpdate

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F64 = torch.float64
EPS = 1e-5
BOTH = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def _same_numbers_every_run():
    torch.manual_seed(20260731)


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
    square error is bounded tightly (a wrong formula, window or state moves it by far more), the largest error loosely."""
    if dtype in (torch.float32, "float32"):
        return _rel(got, want) < 2e-5
    return _rms(got, want) < 1e-2 and _rel(got, want) < 1e-1


def _close_rows(got, want, dtype) -> bool:
    """Whole models.  bfloat16 is bounded row by row: a router's close call may go the other way for a token when its input is
    rounded, which moves that token's logits and little else, while a wrong mechanism moves every row it touches."""
    if dtype in (torch.float32, "float32"):
        return _rel(got, want) < 3e-5
    want = want.double().cpu()
    err = ((got.double().cpu() - want) ** 2).mean(-1).sqrt() / want.abs().max()
    return float(err.median()) < 2e-2 and float((err > 6e-2).double().mean()) <= 0.1


def _bf(t):
    return t.to(torch.bfloat16).to(F64)


def _dev(t, dtype=torch.float32):
    return t.to(DEV, dtype).contiguous()


def _step(lib, cache, slots, q_lens):
    past = [cache.length(s) for s in slots]
    cache.reserve(slots, q_lens)
    return StepContext.for_batch(DEV, StepBatch(slots, past, [[0] * q for q in q_lens], [], cache.block_tables(slots)),
                                 n_compute_units=lib.n_compute_units)


def _place(part, w, dtype):
    specs = part.tensor_specs()
    return {n: _dev(w[n], torch.float32 if specs[n].role == "gain" else dtype) for n in specs}


def _run_mixer(lib, part, x, cuts, dtype, pages=8):
    """The mixer on x [T, E] fed in pieces of the given sizes, through a cache of its own."""
    cache = Cache([part.cache_requests()], 2, 64 * pages, dtype, DEV)
    cache.alloc_slot()                                    # slot 0 stays idle: the sequence lives in slot 1
    slot = cache.alloc_slot()
    outs, at = [], 0
    for n in cuts:
        ctx = _step(lib, cache, [slot], [n])
        outs.append(part.forward(_dev(x[at:at + n], dtype), ctx, cache.view(0, ctx.block_tables)))
        cache.commit([slot], [n])
        at += n
    return torch.cat(outs)


def _config(kind, m, hidden, mlp=None):
    return {"vocab": 4, "width": hidden, "streams": 1, "layers": [{"type": kind, "mixer": m, "mlp": mlp}]}


def _mixer(lib, hidden, kind, m, dtype):
    cfg = GoperaxConfig(vocab=4, width=hidden, streams=1, embedding_scale=1.0, norm_eps=EPS, layers=_config(kind, m, hidden)["layers"],
                        max_positions=2048)
    cfg.check()
    return build_part("mixer", cfg.to_spec().layers[0].mixer, _env(lib, hidden, dtype))


def _weights(kind, hidden, m, seed, part="mix", mlp=None):
    t = P.random_goperax_tensors(_config(kind, m, hidden, mlp), seed)
    return {k[len(f"l0.{part}."):]: v for k, v in t.items() if k.startswith(f"l0.{part}.")}


CUTS = ([200], [63, 1, 1, 2, 61, 72], [130] + [1] * 70, [2] * 5 + [190])


# ---------------------------------------------------------------------------- the two ends
@pytest.mark.parametrize("streams", [1, 3])
@pytest.mark.parametrize("width", [64, 37, 1])
def test_embedding_with_a_scale_and_the_positions_sines_and_cosines(lib, width, streams):
    for dtype in BOTH:
        part = build_part("embedding", PartSpec("table", {"name": "e", "vocab_size": 9, "streams": streams, "scale": 2.75, "waves": 10000.0}),
                          _env(lib, width, dtype))
        table = _bf(torch.randn(9, width, dtype=F64))
        part.load({"e": _dev(table, dtype)})
        # positions at a sequence's start, across a page's border and far beyond what a float32 angle resolves
        pos = torch.tensor([0, 1, 2, 62, 63, 64, 65, 1000, 99991, 1048575])
        ids = torch.tensor([0, 8, 1, 7, 2, 6, 3, 5, 4, 4])

        class Ctx:
            n_tokens, token_ids, tok_pos = len(pos), _dev(ids, torch.int32), _dev(pos, torch.int32)
        x = part.forward(Ctx)
        want = table[ids] * 2.75 + P.wave_vector(pos, width)
        assert x.shape == (streams, len(pos), width)
        for s in range(streams):
            assert _rel(x[s], want) < 3e-7


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width,streams", [(64, 3), (128, 1), (51, 2), (4100, 4), (200, 6), (33, 16), (8, 2)])
def test_norm_of_a_stream_in_copies_behind_an_update_of_the_copies(lib, width, streams, dtype):
    """The update and the norm in one pass: a plain result, the K slices of a product, the outputs of a token's experts with and
    without a shared one; on all rows, and on chosen rows, where the copies stay as they are."""
    tol = 3e-6 if dtype == torch.float32 else 6e-3
    norm = build_part("norm", PartSpec("rmsnorm", {"size": width, "eps": EPS, "names": {"weight": ""}}), _env(lib, width, dtype))
    gain = _bf(torch.randn(width, dtype=F64))
    norm.load({"": _dev(gain)})
    a, b, m = torch.randn(streams, dtype=F64), torch.randn(streams, dtype=F64), torch.randn(streams, streams, dtype=F64)
    a, b, m = a.float().double(), b.float().double(), m.float().double()
    for n in (1, 7, 300):
        x = (2 * torch.randn(streams, n, width, dtype=F64)).float().double()
        plain = lambda copies, coef: P.unit_rms(P.gather_copies(list(copies), coef), EPS) * gain
        assert _rel(norm.forward(_dev(x), None, None, coef=_dev(a)), plain(x, a)) < tol
        assert _rel(norm.forward(_dev(x)), plain(x, torch.ones(streams, dtype=F64))) < tol
        y, terms = torch.randn(n, width, dtype=F64), torch.randn(6, n, width, dtype=F64)
        outputs, weights = torch.randn(n * 3, width, dtype=F64), torch.rand(n * 3, dtype=F64)
        total = (outputs * weights[:, None]).view(n, 3, width).sum(1)
        pairs = lambda shared: ExpertPairs(_dev(outputs), _dev(weights), shared)
        for result, same in ((_dev(y), y), (_dev(terms), terms.sum(0)), (pairs(None), total), (pairs(_dev(y)), total + y),
                             (pairs(_dev(terms)), total + terms.sum(0))):
            update = StreamsUpdate(lib, _dev(m), _dev(b), result, None)
            new = torch.stack(P.rebuild_copies(list(x), b, m, same))
            xd = _dev(x)
            h = norm.forward(xd, update, None, coef=_dev(a))
            assert _rel(xd, new) < 3e-6 and _rel(h, plain(new, a)) < tol
            xd, rows = _dev(x), [n - 1, 0, n // 2]
            h = norm.forward(xd, update, torch.tensor(rows, dtype=torch.int32, device=DEV))
            assert torch.equal(xd, _dev(x)) and _rel(h, plain(new, torch.ones(streams, dtype=F64))[rows]) < tol


# ---------------------------------------------------------------------------- the state-space mixer
def _scan(heads, vdim, state, groups, conv, norm_groups):
    return dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


SCANS = [_scan(4, 24, 40, 2, 3, 2),             # in chunks, with zeros up to the matrix cores' sizes
         _scan(8, 64, 128, 4, 4, 8),            # sizes of a real model's heads
         _scan(6, 16, 32, 3, 2, 1), _scan(2, 128, 16, 1, 4, 4), _scan(3, 8, 256, 1, 4, 3), _scan(2, 72, 64, 2, 5, 1),
         _scan(5, 6, 10, 5, 4, 3),              # sizes off the chunks' grid: token after token
         _scan(1, 1, 1, 1, 1, 1), _scan(4, 32, 24, 1, 1, 16), _scan(2, 160, 8, 2, 6, 5), _scan(3, 4, 300, 3, 2, 2)]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("p", SCANS)
def test_state_space_whole_in_pieces_and_token_by_token(lib, p, dtype):
    hidden = 48
    part = _mixer(lib, hidden, "mamba2", p, dtype)
    w = _weights("mamba2", hidden, p, seed=p["heads"] + p["state"])
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(300, hidden, dtype=F64))
    want = P.mamba2(x, w, p, EPS)
    for cuts in ([300], [63, 1, 1, 2, 61, 172], [230] + [1] * 70, [2] * 5 + [290], [128, 128, 44], [127, 129, 44], [24] * 12 + [12]):
        assert _close(_run_mixer(lib, part, x, cuts, dtype), want, dtype), cuts


def test_the_convolutions_bias_stands_on_its_result_and_its_state_knows_nothing_of_it(lib):
    """One, two and more taps, four channels a thread and one; the state after a step holds the plain inputs."""
    from rbitnet_amd.parts.short_conv import ACT_SILU, ShortConv
    for channels, taps in ((40, 4), (40, 2), (40, 3), (37, 4), (40, 7), (12, 1)):
        env = _env(lib, 8, torch.float32)
        conv = ShortConv(channels, taps, env, residual=False, act=ACT_SILU)
        w, bias, x = torch.randn(channels, taps, dtype=F64), 3 + torch.randn(channels, dtype=F64), torch.randn(70, channels + 8, dtype=F64)
        conv.load(_dev(w))
        req = conv.cache_request("c")
        cache = Cache([[req] if req else []], 2, 64, torch.float32, DEV)
        slot = [cache.alloc_slot(), cache.alloc_slot()][1]
        out, at = [], 0
        for n in (1, 2, 40, 1, 3, 23):
            ctx = _step(lib, cache, [slot], [n])
            state = cache.view(0, ctx.block_tables).states.get("c")
            out.append(conv.forward(_dev(x[at:at + n]), ctx, state, torch.float32, col0=4, bias_out=_dev(bias)))
            cache.commit([slot], [n])
            at += n
            if req:
                kept = torch.cat([torch.zeros(taps - 1, channels, dtype=F64), x[:at, 4:4 + channels]])[-(taps - 1):]
                assert _rel(state[slot], kept) < 1e-6, (taps, at)
        assert _rel(torch.cat(out), P.silu(P.causal_conv(x[:, 4:4 + channels], w, bias))) < 3e-6, (channels, taps)


@pytest.mark.parametrize("dim,vdim,groups", [(128, 64, 2), (32, 32, 1), (64, 128, 4), (256, 16, 2), (40, 72, 4), (8, 8, 4)])
def test_chunks_on_the_matrix_cores_against_the_plain_scan(lib, dim, vdim, groups):
    """The kernels alone: three sequences on top of states that are not zero, piece lengths at and around a chunk.  What the
    state holds afterwards is held to float32 (its operands go in as two bfloat16 numbers each)."""
    heads = 4
    for lens in ((128, 1, 300), (127, 129, 2), (256, 64, 33)):
        t = sum(lens)
        xkq, dt_in = _bf(torch.randn(t, heads * vdim + 2 * groups * dim, dtype=F64)), torch.randn(t, heads + 3, dtype=F64).float().double()
        bias, a_log, d = (v.float().double() for v in (torch.randn(heads, dtype=F64), -2 + torch.randn(heads, dtype=F64), torch.randn(heads, dtype=F64)))
        state, slots = torch.randn(5, heads, vdim, dim, dtype=F64).float().double(), [4, 0, 2]

        class Ctx:
            n_tokens, n_seqs = t, 3
            cu_seqlens = torch.tensor([0, lens[0], lens[0] + lens[1], t], dtype=torch.int32, device=DEV)
        Ctx.slots = torch.tensor(slots, dtype=torch.int32, device=DEV)
        sd, out = _dev(state), torch.empty(t, heads * vdim, device=DEV)
        lib.selective_chunks(_dev(xkq, torch.bfloat16), dim, groups, heads, vdim, _dev(dt_in), 2, _dev(bias), _dev(a_log), _dev(d), sd, Ctx, out)
        single, out1 = _dev(state), torch.empty(t, heads * vdim, device=DEV)
        lib.selective_scan(_dev(xkq), dim, groups, heads, vdim, _dev(dt_in), 2, _dev(bias), _dev(a_log), _dev(d), single, Ctx, out1)
        x, k, q = xkq.split([heads * vdim, groups * dim, groups * dim], 1)
        dt = P.softplus(dt_in[:, 2:2 + heads] + bias)
        at = 0
        for n, slot in zip(lens, slots):
            cut = slice(at, at + n)
            xx, kk, qq, dd = x[cut].view(n, heads, vdim), k[cut].view(n, groups, dim), q[cut].view(n, groups, dim), dt[cut]
            want = P.selective_scan(xx, kk, qq, dd, a_log, d)
            decay = torch.exp(-torch.exp(a_log) * dd.cumsum(0))                        # [n, heads]: of the state in front
            s0 = state[slot].transpose(1, 2)                                           # [head, dim, vdim]
            qh, kh = qq.repeat_interleave(heads // groups, 1), kk.repeat_interleave(heads // groups, 1)
            want = want + torch.matmul(qh.permute(1, 0, 2), s0).permute(1, 0, 2) * decay[:, :, None]
            later = torch.exp(-torch.exp(a_log) * (dd.sum(0) - dd.cumsum(0))) * dd
            end = s0 * decay[-1][:, None, None] + torch.matmul((kh * later[:, :, None]).permute(1, 2, 0).contiguous(), xx.permute(1, 0, 2).contiguous())
            assert _rel(out1[cut], want.reshape(n, -1)) < 2e-5 and _rel(single[slot].transpose(1, 2), end) < 2e-5, (lens, slot)
            assert _rel(sd[slot].transpose(1, 2), end) < 5e-5, (lens, slot)
            assert _rms(out[cut], want.reshape(n, -1)) < 1e-3 and _rel(out[cut], want.reshape(n, -1)) < 1e-2, (lens, slot)
            at += n
        for slot in (1, 3):                                         # nobody's slots stay as they were
            assert torch.equal(sd[slot].cpu(), state[slot].float()) and torch.equal(single[slot].cpu(), state[slot].float())


@pytest.mark.parametrize("dtype", BOTH)
def test_what_the_first_token_wrote_is_read_much_later_beside_another_sequence(lib, dtype):
    """Decays of nearly 1: the state keeps the first token's write for 300 tokens; a second sequence in another slot, fed in
    the same steps at other lengths, keeps its own; a slot that is freed and handed out again starts at zero."""
    hidden, p, t_len = 32, _scan(2, 16, 16, 1, 4, 2), 300
    part = _mixer(lib, hidden, "mamba2", p, dtype)
    w = _weights("mamba2", hidden, p, seed=3)
    w["A_log"] = torch.full((2,), -9.0, dtype=F64)
    w["D"] = torch.zeros(2, dtype=F64)
    part.load(_place(part, w, dtype))
    cache = Cache([part.cache_requests()], 3, 64, dtype, DEV)
    cache.alloc_slot()
    for _ in range(2):
        xs = [_bf(torch.randn(t_len, hidden, dtype=F64)) for _ in range(2)]
        xs[0][0] = xs[0][0] * 12
        wants = [P.mamba2(x, w, p, EPS) for x in xs]
        gone = P.mamba2(torch.cat([torch.zeros(1, hidden, dtype=F64), xs[0][1:]]), w, p, EPS)
        assert _rel(wants[0][-1:], gone[-1:]) > 5e-2                                # the first token still matters at the end
        slots = [cache.alloc_slot(), cache.alloc_slot()]
        outs, at = [[], []], [0, 0]
        for take in ((100, 30), (1, 1), (1, 1), (2, 140), (196, 128)):
            ctx = _step(lib, cache, slots, list(take))
            x = torch.cat([xs[i][at[i]:at[i] + take[i]] for i in range(2)])
            y = part.forward(_dev(x, dtype), ctx, cache.view(0, ctx.block_tables))
            outs[0].append(y[:take[0]])
            outs[1].append(y[take[0]:])
            cache.commit(slots, list(take))
            at = [at[i] + take[i] for i in range(2)]
        assert at == [t_len, t_len]
        for i in range(2):
            assert _close(torch.cat(outs[i]), wants[i], dtype), i
        assert _close(torch.cat(outs[0])[-1], wants[0][-1], dtype)
        for s in slots:
            cache.free_slot(s)


# ---------------------------------------------------------------------------- attention whose values are its keys
def _att(heads, kv_heads, dim, scale, cap=None, window=None):
    out = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale)
    if cap:
        out["softcap"] = cap
    if window:
        out["mask"] = {"size": window}
    return out


ATTENTIONS = [_att(4, 2, 16, 0.3, 12.0, 36), _att(3, 3, 24, 0.2, 50.0, 70), _att(8, 2, 64, 0.12, 20.0, 64), _att(6, 1, 100, 0.1, 30.0, 100),
              _att(1, 1, 6, 0.5, 5.0, 1), _att(2, 1, 128, 0.08, 15.0), _att(5, 5, 7, 0.4, None, 3), _att(34, 2, 32, 0.15, 25.0, 90),
              _att(2, 2, 160, 0.06, 10.0, 50), _att(20, 1, 64, 0.1, None, 65), _att(4, 4, 128, 0.09, 40.0, 129), _att(16, 4, 64, 0.1)]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("p", ATTENTIONS)
def test_attention_whole_in_pieces_and_token_by_token(lib, p, dtype):
    hidden = 64
    part = _mixer(lib, hidden, "attention", p, dtype)
    w = _weights("attention", hidden, p, seed=p["heads"] + p["dim"])
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(200, hidden, dtype=F64))
    want = P.attention(x, w, p)
    for cuts in CUTS:
        got = _run_mixer(lib, part, x, cuts, dtype)
        assert _close(got, want, dtype), cuts
        assert _close(got[:3], want[:3], dtype), cuts            # the first tokens, where the one in the denominator weighs most


def test_the_cache_holds_one_set_of_pages_with_the_keys_as_projected(lib):
    hidden, t_len = 64, 70
    for dtype in BOTH:
        for p in (ATTENTIONS[0], ATTENTIONS[3], ATTENTIONS[6]):
            part = _mixer(lib, hidden, "attention", p, dtype)
            w = _weights("attention", hidden, p, seed=1)
            part.load(_place(part, w, dtype))
            x = _bf(torch.randn(t_len, hidden, dtype=F64))
            cache = Cache([part.cache_requests()], 1, 256, dtype, DEV)
            slot = cache.alloc_slot()
            ctx = _step(lib, cache, [slot], [t_len])
            view = cache.view(0, ctx.block_tables)
            assert view.v_pages.data_ptr() == view.k_pages.data_ptr()
            part.forward(_dev(x, dtype), ctx, view)
            k = (x @ w["k"].T).view(t_len, p["kv_heads"], p["dim"])
            pages = view.block_table[0].tolist()
            for t in (0, 1, 63, 64, t_len - 1):
                row = view.k_pages[pages[t // 64], :, t % 64]
                assert _rel(row[:, :p["dim"]], k[t]) < (1e-5 if dtype == torch.float32 else 1e-2)
                assert float(row[:, p["dim"]:].float().abs().sum()) == 0.0


def _swap(x):
    """The two halves of a row exchanged: W_q is made from W_k so that a query points at the key of the exchanged row."""
    return torch.cat([x[..., x.shape[-1] // 2:], x[..., :x.shape[-1] // 2]], -1)


def _pointing_weights(hidden, p, seed):
    w = _weights("attention", hidden, p, seed)
    d, per = p["dim"], p["heads"] // p["kv_heads"]
    w["q"] = torch.cat([_swap(w["k"][d * (h // per):d * (h // per + 1)]) for h in range(p["heads"])])
    return w


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("window,dim,heads,kv_heads", [(36, 16, 2, 1), (64, 64, 4, 2), (65, 64, 2, 1), (7, 20, 2, 2), (130, 128, 2, 1), (128, 64, 20, 1)])
def test_a_key_that_stands_out_at_every_edge_of_the_window(lib, dtype, window, dim, heads, kv_heads):
    """One earlier token has the key that the query points at: seen as the oldest of the window and as the token just before the
    query, and not one further back; in a prompt and in decoding, at page borders and between them."""
    hidden = 64
    p = _att(heads, kv_heads, dim, 9.0 / dim, 24.0, window)
    w = _pointing_weights(hidden, p, seed=window)
    part = _mixer(lib, hidden, "attention", p, dtype)
    part.load(_place(part, w, dtype))
    for query in (window - 1, window, 64 + window - 1, 64 + window, 2 * 64 + window + 17):
        t_len = query + 4
        for back, seen in ((window - 1, True), (window, False), (1, window > 1), (window + 1, False)):
            at = query - back
            if at < 0:
                continue
            x = _bf(torch.randn(t_len, hidden, dtype=F64))
            x[at] = _swap(x[query])
            q, k = (x @ w["q"].T).view(t_len, heads, dim), (x @ w["k"].T).view(t_len, kv_heads, dim)
            a = P.weights_beside_one(P.scores(q, k, p["scale"], p["softcap"]), P.visible(t_len, window))[:, query, at]
            assert (float(a.min()) > 0.5) if seen else (float(a.max()) == 0.0)           # the edge shows in the plain weights
            want = P.attention(x, w, p)
            for cuts in ([t_len], [query] + [1] * (t_len - query), [at + 1, t_len - at - 1]):
                got = _run_mixer(lib, part, x, cuts, dtype, pages=10)
                assert _close(got, want, dtype), (query, at, cuts)
                assert _close(got[query], want[query], dtype), (query, at, cuts)


@pytest.mark.parametrize("dtype", BOTH)
def test_a_far_key_among_hundreds(lib, dtype):
    """Token 2 has the key that a query 620 tokens later points at."""
    hidden, t_len, p = 64, 640, _att(4, 2, 64, 0.12, 30.0)
    w = _pointing_weights(hidden, p, seed=5)
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    x[2] = _swap(x[622])
    want = P.attention(x, w, p)
    other = x.clone()
    other[2] = _bf(torch.randn(hidden, dtype=F64))
    assert _rel(want[622], P.attention(other, w, p)[622]) > 0.3      # the far token matters to its query
    part = _mixer(lib, hidden, "attention", p, dtype)
    part.load(_place(part, w, dtype))
    for cuts in ([t_len], [600] + [1] * 40, [2, 400, 238]):
        got = _run_mixer(lib, part, x, cuts, dtype, pages=11)
        assert _close(got, want, dtype) and _close(got[622], want[622], dtype), cuts


@pytest.mark.parametrize("dtype", BOTH)
def test_the_cap_and_the_one_beside_the_sum(lib, dtype):
    """Scores far beyond the cap, of either sign: keys that point away leave a weight of next to nothing and an output near zero;
    without a cap of 2 the far larger score would take everything."""
    hidden, t_len = 64, 90
    for dim in (64, 20):
        for sign in (1.0, -1.0):
            p = _att(2, 2, dim, sign * 9.0 / dim, 2.0)
            w = _pointing_weights(hidden, p, seed=dim)
            x = _bf(torch.randn(t_len, hidden, dtype=F64))
            x[:, 32:] = x[:, :32]                                       # every query points at its own key
            want = P.attention(x, w, p)
            wide = P.attention(x, w, dict(p, softcap=50.0))
            assert _rel(wide, want) > 0.3
            part = _mixer(lib, hidden, "attention", p, dtype)
            part.load(_place(part, w, dtype))
            for cuts in ([t_len], [30] + [1] * 60):
                assert _close(_run_mixer(lib, part, x, cuts, dtype), want, dtype), (dim, sign, cuts)


@pytest.mark.parametrize("splits", [1, 3, 16])
@pytest.mark.parametrize("window", [None, 500])
def test_long_decoding_with_the_pages_dealt_to_several_workgroups(lib, window, splits):
    """1,100 tokens, the last 60 one by one; the number of shares forced, as a long context would choose it."""
    from rbitnet_amd.engine import context as C
    hidden, t_len = 64, 1100
    p = _att(8, 2, 64, 0.05, 30.0, window)
    w = _weights("attention", hidden, p, seed=11)
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    want = P.attention(x, w, p)
    part = _mixer(lib, hidden, "attention", p, torch.bfloat16)
    part.load(_place(part, w, torch.bfloat16))
    C.FORCED_DECODE_SPLITS = splits
    try:
        got = _run_mixer(lib, part, x, [t_len - 60] + [1] * 60, torch.bfloat16, pages=20)
    finally:
        C.FORCED_DECODE_SPLITS = None
    assert _close(got, want, torch.bfloat16) and _close(got[-60:], want[-60:], torch.bfloat16)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("kind", ["attention", "mamba2"])
def test_several_sequences_that_go_on_at_unequal_lengths(lib, kind, dtype):
    """Three sequences in one step, on top of unequal pasts, against each alone; slots, pages and states are then freed and used
    again by other sequences."""
    hidden = 64
    p = _att(8, 2, 64, 0.12, 30.0, 100) if kind == "attention" else _scan(4, 32, 32, 2, 4, 2)
    w = _weights(kind, hidden, p, seed=4)
    part = _mixer(lib, hidden, kind, p, dtype)
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
            y = part.forward(_dev(torch.cat([xs[i][at[i]:at[i] + n] for i, n in zip(live, take)]), dtype), ctx, cache.view(0, ctx.block_tables))
            off = 0
            for i, n in zip(live, take):
                outs[i].append(y[off:off + n])
                off += n
                at[i] += n
            cache.commit([slots[i] for i in live], take)
        for i in range(3):
            assert _close(torch.cat(outs[i]), P.MIXERS[kind](xs[i], w, p, EPS), dtype), (lens, i)
        for s in slots:
            cache.free_slot(s)
        cache.check()


# ---------------------------------------------------------------------------- feed-forwards
@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("hidden,ff,t_len", [(64, 128, 70), (64, 128, 8), (48, 51, 5), (256, 1024, 300), (50, 31, 33)])
def test_dense_with_the_squared_relu(lib, dtype, hidden, ff, t_len):
    part = build_part("feed_forward", PartSpec("dense_act", {"intermediate_size": ff, "activation": "squared_relu"}), _env(lib, hidden, dtype))
    w = _weights("attention", hidden, ATTENTIONS[0], ff, "mlp", {"kind": "dense", "ff": ff})
    part.load(_place(part, w, dtype))
    x = _bf(2 * torch.randn(t_len, hidden, dtype=F64))
    assert _close(part.forward(_dev(x, dtype)), P.plain_unit(x, w["up"], w["down"]), dtype)


EXPERTS = [(64, 32, 4, 2, 70, 48), (48, 24, 7, 3, 33, 20), (32, 16, 1, 1, 9, None), (128, 64, 16, 4, 300, 128), (50, 31, 5, 5, 20, 17),
           (64, 96, 130, 6, 40, None), (224, 96, 11, 3, 1, 32), (96, 64, 9, 2, 32, 1), (64, 32, 70, 64, 5, None)]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("hidden,ff,experts,top,t_len,shared", EXPERTS)
def test_experts_without_gates_beside_a_shared_one(lib, dtype, hidden, ff, experts, top, t_len, shared):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
    part = build_part("feed_forward", GoperaxConfig._feed_forward(mlp), _env(lib, hidden, dtype))
    w = _weights("attention", hidden, ATTENTIONS[0], experts + top, "mlp", mlp)
    part.load(_place(part, w, dtype))
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    want = P.experts(x, w, mlp)
    total, pairs = part.forward(_dev(x, dtype)), part.forward(_dev(x, dtype), pairs=True)
    summed = (pairs.outputs.view(t_len, top, hidden) * pairs.weights.view(t_len, top, 1)).sum(1)
    if shared:
        summed = summed + pairs.shared
    assert _close(total, want, dtype) and _close(summed, want, dtype)
    assert torch.allclose(pairs.weights.view(t_len, top).sum(1), torch.ones(t_len, device=DEV), atol=1e-5)
    tol = 1e-5 if dtype == torch.float32 else 2e-3              # (a shared expert's product rounds its units to the compute dtype)
    alone = torch.cat([part.forward(_dev(x[i:i + 1], dtype)) for i in range(min(t_len, 6))])      # the same whatever else a step holds
    assert _rel(alone, total[:len(alone)].double().cpu()) < tol
    for n in (2, 16, 17, 48, 64, 65):                            # the kernels for few tokens and those for many add up alike
        if n < t_len:
            assert _rel(part.forward(_dev(x[:n], dtype)), total[:n].double().cpu()) < tol, n


@pytest.mark.parametrize("hidden,ff,experts,top,t_len", [(128, 64, 6, 2, 300), (64, 192, 3, 3, 900), (192, 128, 130, 4, 70), (64, 64, 1, 1, 65),
                                                         (256, 320, 5, 1, 700)])
def test_experts_on_the_dense_products_tiles_give_what_the_routed_kernels_give(lib, hidden, ff, experts, top, t_len, monkeypatch):
    """Runs padded to 64, 128 and 256 rows, some of them empty, with one expert that nearly every token chooses: bit for bit the
    same pairs."""
    from rbitnet_amd.parts import routed as R
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    part = build_part("feed_forward", GoperaxConfig._feed_forward(mlp), _env(lib, hidden, torch.bfloat16))
    w = _weights("attention", hidden, ATTENTIONS[0], experts + ff, "mlp", mlp)
    x = _bf(torch.randn(t_len, hidden, dtype=F64))
    x[:, 0] = 3.0
    w["router"][0, 0] = 3.0
    part.load(_place(part, w, torch.bfloat16))
    assert part.tiled
    want, h = P.experts(x, w, mlp), _dev(x, torch.bfloat16)
    part.tiled = False
    plain = part.forward(h, pairs=True)
    part.tiled = True
    for unit in (64, 128, 256):
        monkeypatch.setattr(R, "tile_rows", lambda pairs, n: unit)
        got = part.forward(h, pairs=True)
        assert torch.equal(got.outputs, plain.outputs) and torch.equal(got.weights, plain.weights), unit
        assert _close(part.forward(h), want, torch.bfloat16), unit


# ---------------------------------------------------------------------------- whole models
def _moe(ff, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def _dense(ff):
    return {"kind": "dense", "ff": ff}


# everything different from layer to layer
MODEL_A = {"architecture": "Goperax", "vocab": 96, "width": 64, "streams": 4, "embedding": {"scale": 3.5}, "norm": {"eps": 1e-5},
           "loop": {"start": 1, "stop": 4, "times": 2}, "layers": [
               {"type": "attention", "mixer": _att(4, 2, 16, 0.3, 12.0, 44), "mlp": _moe(24, 5, 2, 40)},
               {"type": "mamba2", "mixer": _scan(4, 24, 40, 2, 3, 2), "mlp": None},
               {"type": "attention", "mixer": _att(3, 3, 24, 0.2, 30.0, 9), "mlp": _dense(72)},
               {"type": "mamba2", "mixer": _scan(3, 16, 8, 1, 4, 3), "mlp": _moe(40, 3, 3)},
               {"type": "attention", "mixer": _att(6, 1, 8, 0.3, 50.0), "mlp": None},
               {"type": "mamba2", "mixer": _scan(2, 20, 12, 2, 2, 1), "mlp": _moe(16, 8, 1, 24)}]}
# values that a model may happen to make equal or 1
MODEL_B = {"architecture": "Goperax", "vocab": 50, "width": 32, "streams": 1, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-6},
           "loop": {"start": 0, "stop": 1, "times": 1}, "layers": [
               {"type": "mamba2", "mixer": _scan(1, 32, 32, 1, 1, 1), "mlp": _moe(32, 1, 1, 32)},
               {"type": "attention", "mixer": _att(1, 1, 32, 1.0, 1.0, 1), "mlp": _dense(32)}]}
# sizes on the matrix cores' grid
MODEL_C = {"architecture": "Goperax", "vocab": 320, "width": 128, "streams": 2, "embedding": {"scale": 8.0}, "norm": {"eps": 1e-5},
           "loop": {"start": 0, "stop": 2, "times": 3}, "layers": [
               {"type": "mamba2", "mixer": _scan(8, 32, 64, 2, 4, 4), "mlp": _moe(64, 6, 2, 64)},
               {"type": "attention", "mixer": _att(8, 2, 64, 0.1, 30.0, 128), "mlp": _moe(128, 4, 2, 96)},
               {"type": "mamba2", "mixer": _scan(4, 64, 128, 1, 4, 1), "mlp": _dense(256)},
               {"type": "attention", "mixer": _att(4, 4, 128, 0.08, 25.0, 70), "mlp": _moe(64, 8, 3)}]}
# sizes off every grid
MODEL_D = {"architecture": "Goperax", "vocab": 37, "width": 51, "streams": 5, "embedding": {"scale": 2.0}, "norm": {"eps": 1e-4}, "layers": [
    {"type": "mamba2", "mixer": _scan(5, 7, 11, 5, 6, 7), "mlp": _moe(31, 3, 2, 9)},
    {"type": "attention", "mixer": _att(3, 1, 10, 0.3, 8.0, 3), "mlp": _dense(29)},
    {"type": "attention", "mixer": _att(5, 5, 6, 0.4, None, 67), "mlp": _moe(7, 5, 1)},
    {"type": "mamba2", "mixer": _scan(3, 5, 3, 1, 2, 1), "mlp": None}]}
MODELS = {"A": (MODEL_A, 114), "B": (MODEL_B, 22), "C": (MODEL_C, 23), "D": (MODEL_D, 24)}
_TMP = tempfile.TemporaryDirectory(prefix="goperax_models_")
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
        tensors = P.random_goperax_tensors(cfg, seed)
        folder = os.path.join(_TMP.name, name)
        _write(folder, cfg, tensors)
        _MADE[name] = (folder, P.PlainGoperax(copy.deepcopy(cfg), tensors))
    return _MADE[name]


def _tokens(name, n, seed):
    g = torch.Generator().manual_seed(100 * seed + n)
    return torch.randint(0, MODELS[name][0]["vocab"], (n,), generator=g).tolist()


def _engine(name, dtype, **kw):
    import rbitnet_amd
    return rbitnet_amd.Engine.load_path(_model(name)[0], dtype=dtype, max_seq_len=1024, **kw)


@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_every_layer_of_a_model_against_the_plain_stream(name):
    """The sum of the copies after every layer that runs (float32), so that a fault names its layer."""
    from rbitnet_amd.parts import hyper as H
    eng = _engine(name, "float32", max_tokens=64 * 4, max_batch=1)
    toks = _tokens(name, 90, 4)
    want = _model(name)[1].streams(toks)
    seen = []
    orig = H.HyperBlock.forward

    def traced(self, x, pending, ctx, view, next_norm=None):
        out = orig(self, x, pending, ctx, view, next_norm)
        mix, b, y, weights, extra = (None if t is None else t.double().cpu() for t in out.term_parts())
        if weights is not None:
            y = (y.view(x.shape[1], -1, x.shape[2]) * weights.view(x.shape[1], -1, 1)).sum(1)
        y = y.sum(0) if y.dim() == 3 else y
        if extra is not None:
            y = y + (extra.sum(0) if extra.dim() == 3 else extra)
        seen.append(sum(P.rebuild_copies(list(x.double().cpu()), b, mix, y)))        # what the next norm still has to do
        return out

    H.HyperBlock.forward = traced
    try:
        slot = eng.alloc_slot()
        eng.use_plans = False
        eng.step([(slot, toks)], "last")
    finally:
        H.HyperBlock.forward = orig
    assert len(seen) == len(want) == len(eng.spec.schedule)
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
    new requests take the freed slots, pages and states.  Every request's logits are those it has alone."""
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
    implementation's greedy tokens for a batch of unequal prompts, past every layer's window."""
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
        margin = (1e-4 if dtype == "float32" else 0.04) * float(logits.abs().max())
        clear = (top2.values[:, 0] - top2.values[:, 1]) > margin          # a tie within rounding may go either way
        same = sum(1 for g, t, c in zip(top2.indices[:, 0].tolist(), r.tokens, clear.tolist()) if c and g == t)
        assert same >= (1.0 if dtype == "float32" else 0.95) * int(clear.sum())
        assert int(clear.sum()) > (0.9 if dtype == "float32" else 0.4) * n
    assert eng.stats["decode_tokens"] > 0 and eng.model.graph_safe and eng.model.plan_safe


def _random_config(rng):
    """A model whose every size, constant and layer order is drawn: what no hand-made model thought of."""
    def mixer(kind):
        if kind == "mamba2":
            groups, per, vdim = rng.choice([1, 2, 3]), rng.choice([1, 2, 3, 4]), rng.choice([4, 8, 16, 20, 24, 32, 64, 128])
            inner = groups * per * vdim
            return _scan(groups * per, vdim, rng.choice([4, 8, 16, 24, 32, 64, 128, 256]), groups, rng.choice([1, 2, 3, 4, 5, 8]),
                         rng.choice([n for n in (1, 2, 3, 4, 6, 8) if inner % n == 0]))
        kvh, group = rng.choice([1, 2, 3, 4]), rng.choice([1, 2, 3, 4, 8, 20])
        return _att(kvh * group, kvh, rng.choice([8, 16, 20, 32, 48, 64, 96, 128]), rng.choice([0.05, 0.1, 0.2]), rng.choice([10.0, 30.0, 50.0]),
                    rng.choice([None, 1, 7, 16, 36, 64, 65, 100, 128, 200]))

    layers = []
    for _ in range(rng.choice([2, 3, 4, 5])):
        n, x = rng.choice([1, 2, 5, 8, 12, 20]), rng.random()
        mlp = None if x < 0.15 else _dense(rng.choice([16, 48, 100, 256])) if x < 0.4 else \
            _moe(rng.choice([8, 16, 40, 64, 96]), n, rng.randint(1, min(n, 4)), rng.choice([None, 8, 24, 64]))
        kind = rng.choice(["mamba2", "attention"])
        layers.append({"type": kind, "mixer": mixer(kind), "mlp": mlp})
    out = {"architecture": "Goperax", "vocab": rng.choice([37, 96, 300, 450]), "width": rng.choice([32, 48, 64, 96, 128, 160, 320]),
           "streams": rng.choice([1, 2, 3, 4, 5]), "embedding": {"scale": rng.choice([1.0, 5.0, 12.0])}, "norm": {"eps": rng.choice([1e-5, 1e-6])},
           "layers": layers}
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        out["loop"] = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.choice([1, 2, 3])}
    return out


@pytest.mark.parametrize("seed", list(range(60, 72)))
def test_models_drawn_at_random_whole_in_pieces_decoded_and_batched(seed, tmp_path):
    import random
    import rbitnet_amd
    cfg = _random_config(random.Random(seed))
    tensors = P.random_goperax_tensors(cfg, seed)
    oracle = P.PlainGoperax(copy.deepcopy(cfg), tensors)
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
