"""A plain, slow float64 implementation of the Goperax decoder, one function per mechanism, whole sequences only
(no cache, no state, no batches): the oracle of the tests.  It shares no code with the package.

Notation: T tokens, E width; weights are [out, in] and applied as x @ W.T.  The residual stream is a list of S copies of the
embedding's output; a sublayer f with its own mixing numbers (a [S], b [S], M [S, S]) does
    y = f(n(sum_s a_s x_s));   x_t <- sum_s M[s, t] x_s + b_t y      for all t from the old copies
once for the mixer and once for the feed-forward of every layer.  What comes out is the sum of the copies.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional

import torch

F64 = torch.float64


# ---------------------------------------------------------------- small things
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def squared_relu(x):
    return torch.clamp(x, min=0.0) ** 2


def wave_vector(positions, width: int, base: float = 10000.0):
    """positions [T] -> [T, width]: numbers 2i and 2i + 1 are the sine and the cosine of position * base^(-2i / width)."""
    out = torch.zeros(len(positions), width, dtype=F64)
    for j in range(width):
        angle = positions.to(F64) * base ** (-2.0 * (j // 2) / width)
        out[:, j] = torch.sin(angle) if j % 2 == 0 else torch.cos(angle)
    return out


def embedding(tokens: List[int], table, scale: float):
    return table[torch.tensor(tokens)] * scale + wave_vector(torch.arange(len(tokens)), table.shape[1])


# ---------------------------------------------------------------- the stream in several copies
def gather_copies(copies, a):
    return sum(a[s] * copies[s] for s in range(len(copies)))


def rebuild_copies(copies, b, mix, y):
    n = len(copies)
    return [sum(mix[s, t] * copies[s] for s in range(n)) + b[t] * y for t in range(n)]


# ---------------------------------------------------------------- the state-space mixer
def causal_conv(x, taps, bias):
    """x [T, C], taps [C, K]: y_t = bias + sum_d taps[:, K - 1 - d] x_(t - d), zeros before the start."""
    t_len, k = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(k - 1, x.shape[1], dtype=x.dtype), x])
    return bias + sum(taps[:, j] * padded[j:j + t_len] for j in range(k))


def selective_scan(x, b, c, dt, a_log, d):
    """x [T, H, V], b and c [T, G, N], dt [T, H], a_log and d [H]: with head h on group h // (H / G),
    S <- exp(-exp(a_log_h) dt) S + dt b x^T;  y = S^T c + d_h x, one token after another -> [T, H, V]"""
    t_len, heads, v = x.shape
    per = heads // b.shape[1]
    state = torch.zeros(heads, b.shape[2], v, dtype=x.dtype)
    out = torch.zeros(t_len, heads, v, dtype=x.dtype)
    for t in range(t_len):
        bb, cc = b[t].repeat_interleave(per, 0), c[t].repeat_interleave(per, 0)
        keep = torch.exp(-torch.exp(a_log) * dt[t])
        state = keep[:, None, None] * state + dt[t][:, None, None] * bb[:, :, None] * x[t][:, None, :]
        out[t] = (state * cc[:, :, None]).sum(1) + d[:, None] * x[t]
    return out


def gated_group_norm(y, z, weight, groups: int, eps: float):
    """The gate first, then a norm of each of `groups` equal parts of the row, then the weight."""
    g = y * silu(z)
    return unit_rms(g.view(g.shape[0], groups, -1), eps).reshape(g.shape) * weight


def mamba2(h, w: Dict[str, torch.Tensor], p: Dict, eps: float):
    t_len = h.shape[0]
    heads, v, n, g = p["heads"], p["vdim"], p["state"], p["groups"]
    inner = heads * v
    z, xbc, dt = torch.split(h @ w["in"].T, [inner, inner + 2 * g * n, heads], dim=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, b, c = torch.split(xbc, [inner, g * n, g * n], dim=1)
    y = selective_scan(x.reshape(t_len, heads, v), b.reshape(t_len, g, n), c.reshape(t_len, g, n),
                       softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    return gated_group_norm(y.reshape(t_len, inner), z, w["norm"], p["norm_groups"], eps) @ w["o"].T


# ---------------------------------------------------------------- attention
def visible(t_len: int, window: Optional[int] = None):
    """[T, T] bool: 0 <= i - j, and with a window also i - j < window."""
    back = torch.arange(t_len)[:, None] - torch.arange(t_len)[None, :]
    return (back >= 0) if window is None else (back >= 0) & (back < window)


def capped(s, cap: Optional[float]):
    return s if cap is None else cap * torch.tanh(s / cap)


def scores(q, k, scale: float, cap: Optional[float]):
    """q [T, H, D], k [T, G, D] -> [H, T, T]"""
    kk = k.repeat_interleave(q.shape[1] // k.shape[1], 1)
    return capped(torch.matmul(q.transpose(0, 1), kk.permute(1, 2, 0)) * scale, cap)


def weights_beside_one(s, seen):
    """exp(s_j) / (1 + sum_j exp(s_j)) over the visible keys."""
    s = s.masked_fill(~seen, -math.inf)
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention(h, w: Dict[str, torch.Tensor], p: Dict, eps: float = 0.0):
    t_len = h.shape[0]
    q = (h @ w["q"].T).view(t_len, p["heads"], p["dim"])
    k = (h @ w["k"].T).view(t_len, p["kv_heads"], p["dim"])
    mask = p.get("mask")
    a = weights_beside_one(scores(q, k, p["scale"], p.get("softcap")), visible(t_len, None if mask is None else mask["size"]))
    o = torch.matmul(a, k.repeat_interleave(p["heads"] // p["kv_heads"], 1).transpose(0, 1)).transpose(0, 1)
    return o.reshape(t_len, -1) @ w["o"].T


MIXERS = {"mamba2": mamba2, "attention": attention}


# ---------------------------------------------------------------- feed-forward
def plain_unit(x, up, down):
    return squared_relu(x @ up.T) @ down.T


def route(h, router, top: int):
    """-> (chosen [T, top], weights [T, top]): the largest of the softmax over all, divided by their sum."""
    best = torch.softmax(h @ router.T, dim=-1).topk(top, dim=-1)
    return best.indices, best.values / (best.values.sum(-1, keepdim=True) + 1e-20)


def experts(h, w: Dict[str, torch.Tensor], p: Dict):
    chosen, weights = route(h, w["router"], p["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(p["router"]["experts"]):
        t, k = torch.nonzero(chosen == e, as_tuple=True)
        if len(t):
            out.index_add_(0, t, plain_unit(h[t], w[f"e{e}.up"], w[f"e{e}.down"]) * weights[t, k][:, None])
    if p.get("shared") is not None:
        out = out + plain_unit(h, w["shared.up"], w["shared.down"])
    return out


def feed_forward(h, w: Dict[str, torch.Tensor], p: Dict):
    return plain_unit(h, w["up"], w["down"]) if p["kind"] == "dense" else experts(h, w, p)


# ---------------------------------------------------------------- the model
def sub(w: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def run_order(cfg: Dict) -> List[int]:
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


class PlainGoperax:
    def __init__(self, config: Dict, tensors: Dict[str, torch.Tensor]):
        self.cfg = config
        self.w = {k: v.to(F64) for k, v in tensors.items()}
        self.eps = float(config["norm"]["eps"])

    @classmethod
    def from_folder(cls, folder: str) -> "PlainGoperax":
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            cfg = json.load(f)
        return cls(cfg, load_file(os.path.join(folder, "model.safetensors")))

    def norm(self, name: str, x):
        return unit_rms(x, self.eps) * self.w[name]

    def layer(self, i: int, copies):
        layer, p = self.cfg["layers"][i], f"l{i}."
        subs = [(1, lambda h: MIXERS[layer["type"]](h, sub(self.w, p + "mix."), layer["mixer"], self.eps))]
        if layer.get("mlp") is not None:
            subs.append((2, lambda h: feed_forward(h, sub(self.w, p + "mlp."), layer["mlp"])))
        for q, f in subs:
            hc = sub(self.w, f"{p}hc{q}.")
            y = f(self.norm(f"{p}norm{q}", gather_copies(copies, hc["in"])))
            copies = rebuild_copies(copies, hc["out"], hc["mix"], y)
        return copies

    def streams(self, tokens: List[int]) -> List[torch.Tensor]:
        """The sum of the copies after every layer that runs."""
        x = embedding(tokens, self.w["embed"], float(self.cfg["embedding"]["scale"]))
        copies = [x] * int(self.cfg["streams"])
        out = []
        for i in run_order(self.cfg):
            copies = self.layer(i, copies)
            out.append(sum(copies))
        return out

    def logits(self, tokens: List[int]) -> torch.Tensor:
        return self.norm("final.norm", self.streams(tokens)[-1]) @ self.w["embed"].T


# ---------------------------------------------------------------- random models for the tests
def tensor_shapes(cfg: Dict) -> Dict[str, tuple]:
    """Name -> shape of every tensor of a model."""
    e, s = cfg["width"], cfg["streams"]
    out = {"embed": (cfg["vocab"], e), "final.norm": (e,)}
    for i, layer in enumerate(cfg["layers"]):
        m, q = layer["mixer"], f"l{i}.mix."
        if layer["type"] == "mamba2":
            h, inner = m["heads"], m["heads"] * m["vdim"]
            ch = inner + 2 * m["groups"] * m["state"]
            out.update({q + "in": (inner + ch + h, e), q + "conv": (ch, m["conv"]), q + "conv.b": (ch,), q + "dt_bias": (h,),
                        q + "A_log": (h,), q + "D": (h,), q + "norm": (inner,), q + "o": (e, inner)})
        else:
            out.update({q + "q": (m["heads"] * m["dim"], e), q + "k": (m["kv_heads"] * m["dim"], e),
                        q + "o": (e, m["heads"] * m["dim"])})
        mlp, q = layer.get("mlp"), f"l{i}.mlp."
        if mlp is not None and mlp["kind"] == "dense":
            out.update({q + "up": (mlp["ff"], e), q + "down": (e, mlp["ff"])})
        elif mlp is not None:
            n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            out[q + "router"] = (n, e)
            for x in range(n):
                out.update({f"{q}e{x}.up": (ff, e), f"{q}e{x}.down": (e, ff)})
            if mlp.get("shared") is not None:
                out.update({q + "shared.up": (mlp["shared"]["ff"], e), q + "shared.down": (e, mlp["shared"]["ff"])})
        for k in (1, 2) if mlp is not None else (1,):
            out.update({f"l{i}.norm{k}": (e,), f"l{i}.hc{k}.in": (s,), f"l{i}.hc{k}.out": (s,), f"l{i}.hc{k}.mix": (s, s)})
    return out


def random_goperax_tensors(cfg: Dict, seed: int) -> Dict[str, torch.Tensor]:
    """Weights that bfloat16 holds exactly, so that the oracle and a model loaded from a bfloat16 file see the same numbers.
    Sizes are chosen so that every mechanism matters at tiny widths."""
    g = torch.Generator().manual_seed(seed)
    rand = lambda shape: torch.randn(shape, generator=g)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if "norm" in last:
            t = 1.0 + 0.2 * rand(shape)
        elif last == "in" and ".hc" in name:
            t = (1.0 + 0.3 * rand(shape)) / shape[0]
        elif last == "out":
            t = 0.6 + 0.4 * rand(shape)
        elif last == "mix" and ".hc" in name:
            t = 0.8 * torch.eye(shape[0]) + 0.15 * rand(shape)
        elif last == "A_log":
            t = -1.5 + 1.2 * rand(shape)
        elif last == "dt_bias":
            t = -1.0 + rand(shape)
        elif last == "D":
            t = 1.0 + 0.5 * rand(shape)
        elif last == "b":
            t = 0.3 * rand(shape)
        elif last == "conv":
            t = rand(shape) * 0.7
        elif name == "embed":
            t = rand(shape) * 0.5
        elif ".mix.q" in name or ".mix.k" in name:
            t = rand(shape) * (1.6 / math.sqrt(shape[-1]))
        else:
            t = rand(shape) * (0.9 / math.sqrt(shape[-1]))
        out[name] = t.to(torch.bfloat16).to(F64)
    return out
