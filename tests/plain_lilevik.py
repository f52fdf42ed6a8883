"""A plain, slow float64 implementation of the Lilevik decoder, one function per mechanism, whole sequences only
(no cache, no state, no batches): the oracle of the tests.  It shares no code with the package.

Notation: T tokens, E width; weights are [out, in] and applied as x @ W.T.  A layer is
    x <- x + n1b(mixer(n1(x)));  x <- x + n2b(experts(n2(x)))
with norms in front of and behind both sublayers, each of them tanh(alpha x) w + b, number by number.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional

import torch

F64 = torch.float64


# ---------------------------------------------------------------- small things
def tanh_norm(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


def frequencies(dims: int, base: float, scaling: Optional[Dict] = None):
    """(f, m): f_i = base^(-2i/dims), i < dims/2, and the factor m on cosine and sine.  With `scaling` {factor, original,
    fast, slow}: a pair that turns `fast` times and more over `original` positions keeps its frequency, one that turns
    `slow` times and less has it divided by factor, a ramp over the pair's index lies between; m = 0.1 ln(factor) + 1."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return torch.tensor(f, dtype=F64), 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index_of(float(scaling["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(factor) + 1.0


def rotate(x, f, m: float = 1.0, first_pos: int = 0):
    """x [T, H, D]: of the first 2 len(f) numbers of every head 2i and 2i + 1 are a pair, turned by position * f_i and
    multiplied by m; the rest pass."""
    t_len, dims = x.shape[0], 2 * f.shape[0]
    a = (torch.arange(t_len, dtype=F64) + first_pos)[:, None] * f[None, :]
    cos, sin = m * torch.cos(a)[:, None, :], m * torch.sin(a)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    r = torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1).reshape(*x.shape[:-1], dims)
    return torch.cat([r, x[..., dims:]], dim=-1)


def visible(t_len: int, chunk: Optional[int] = None):
    """[T, T] bool: j <= i, and with a chunk also floor(i / chunk) = floor(j / chunk)."""
    i = torch.arange(t_len)[:, None]
    j = torch.arange(t_len)[None, :]
    seen = j <= i
    if chunk is not None:
        seen = seen & (torch.div(i, chunk, rounding_mode="floor") == torch.div(j, chunk, rounding_mode="floor"))
    return seen


def scores(q, k, scale: float):
    """q [T, H, D], k [T, G, D] -> [H, T, T]"""
    kk = k.repeat_interleave(q.shape[1] // k.shape[1], 1)
    return torch.matmul(q.transpose(0, 1), kk.permute(1, 2, 0)) * scale


def sigmoid_weights(q, k, scale: float, bias, seen):
    """Every visible key's weight by itself: they are not normalised over the keys."""
    return torch.sigmoid(scores(q, k, scale) + bias[:, None, None]) * seen.to(F64)


def softmax_weights(q, k, scale: float, seen):
    return torch.softmax(scores(q, k, scale).masked_fill(~seen, -math.inf), dim=-1)


def weighted(weights, v):
    """weights [H, T, T], v [T, G, Dv] -> [T, H, Dv]"""
    vv = v.repeat_interleave(weights.shape[0] // v.shape[1], 1)
    return torch.matmul(weights, vv.transpose(0, 1)).transpose(0, 1)


# ---------------------------------------------------------------- mixers
def latent_attention(h, w: Dict[str, torch.Tensor], p: Dict, eps: float):
    t_len = h.shape[0]
    heads, d, r, dv, rank = p["heads"], p["dim"], p["rot_dim"], p["vdim"], p["kv_rank"]
    f, m = frequencies(r, p["rot"]["base"], p["rot"].get("scaling")) if r else (torch.zeros(0, dtype=F64), 1.0)
    cq = unit_rms(h @ w["dq"].T, eps) * w["dq.norm"]
    q = (cq @ w["uq"].T).view(t_len, heads, d + r)
    down = h @ w["dkv"].T
    c = unit_rms(down[:, :rank], eps) * w["dkv.norm"]
    k_rot = rotate(down[:, rank:].view(t_len, 1, r), f, m).expand(t_len, heads, r)
    kk = torch.cat([(c @ w["uk"].T).view(t_len, heads, d), k_rot], dim=-1)
    qq = torch.cat([q[..., :d], rotate(q[..., d:], f, m)], dim=-1)
    v = (c @ w["uv"].T).view(t_len, heads, dv)
    o = weighted(softmax_weights(qq, kk, p["scale"], visible(t_len)), v)
    return o.reshape(t_len, heads * dv) @ w["o"].T


def prepared_heads(h, w: Dict[str, torch.Tensor], p: Dict, eps: float):
    """q, k, v as attention reads them: norms over the whole of q and of k, rotation, every value head divided by its
    root mean square."""
    t_len = h.shape[0]
    heads, groups, d, dv = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    q = (unit_rms(h @ w["q"].T, eps) * w["q.norm"]).view(t_len, heads, d)
    k = (unit_rms(h @ w["k"].T, eps) * w["k.norm"]).view(t_len, groups, d)
    v = unit_rms((h @ w["v"].T).view(t_len, groups, dv), eps)
    rot = p.get("rot")
    if rot and rot["dims"]:
        f, m = frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        q, k = rotate(q, f, m), rotate(k, f, m)
    return q, k, v


def attention(h, w: Dict[str, torch.Tensor], p: Dict, eps: float):
    t_len = h.shape[0]
    q, k, v = prepared_heads(h, w, p, eps)
    mask = p.get("mask")
    seen = visible(t_len, None if mask is None else mask["size"])
    o = weighted(sigmoid_weights(q, k, p["scale"], w["pb"], seen), v)
    return o.reshape(t_len, -1) @ w["o"].T


def decaying_sum(q, k, v, decay):
    """q, k [T, H, D], v [T, H, Dv], decay [H]: S <- decay S + k v^T, o = S^T q, one token after another -> [T, H, Dv]"""
    t_len, heads, d = q.shape
    state = torch.zeros(heads, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for t in range(t_len):
        state = decay[:, None, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (state * q[t][:, :, None]).sum(1)
    return out


def lightning(h, w: Dict[str, torch.Tensor], p: Dict, eps: float):
    t_len = h.shape[0]
    heads, d, dv = p["heads"], p["dim"], p["vdim"]
    q, k = silu(h @ w["q"].T).view(t_len, heads, d), silu(h @ w["k"].T).view(t_len, heads, d)
    v = silu(h @ w["v"].T).view(t_len, heads, dv)
    o = decaying_sum(q, k, v, torch.tensor(p["decay"], dtype=F64)).reshape(t_len, heads * dv)
    return (unit_rms(o, eps) * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


MIXERS = {"latent_attention": latent_attention, "attention": attention, "lightning": lightning}


# ---------------------------------------------------------------- feed-forward
def route(h, router, bias, top: int):
    """-> (chosen [T, top], weights [T, top]): the largest logits, and the softmax over these alone."""
    z = h @ router.T + bias
    best = z.topk(top, dim=-1)
    return best.indices, torch.softmax(best.values, dim=-1)


def expert(x, gate, up, down):
    return (silu(x @ gate.T) * (x @ up.T)) @ down.T


def experts(h, w: Dict[str, torch.Tensor], p: Dict):
    chosen, weights = route(h, w["router"], w["router.b"], p["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(p["router"]["experts"]):
        t, k = torch.nonzero(chosen == e, as_tuple=True)
        if len(t):
            y = expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
            out.index_add_(0, t, y * weights[t, k][:, None])
    return out


# ---------------------------------------------------------------- the model
def sub(w: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


class PlainLilevik:
    def __init__(self, config: Dict, tensors: Dict[str, torch.Tensor]):
        self.cfg = config
        self.w = {k: v.to(F64) for k, v in tensors.items()}
        self.eps = float(config["norm"]["eps"])

    @classmethod
    def from_folder(cls, folder: str) -> "PlainLilevik":
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            cfg = json.load(f)
        return cls(cfg, load_file(os.path.join(folder, "model.safetensors")))

    def norm(self, name: str, x):
        return tanh_norm(x, self.w[name + ".alpha"], self.w[name], self.w[name + ".b"])

    def layer(self, i: int, x):
        layer, p = self.cfg["layers"][i], f"l{i}."
        y = MIXERS[layer["type"]](self.norm(p + "norm1", x), sub(self.w, p + "mix."), layer["mixer"], self.eps)
        x = x + self.norm(p + "norm1b", y)
        if layer.get("mlp") is not None:
            y = experts(self.norm(p + "norm2", x), sub(self.w, p + "mlp."), layer["mlp"])
            x = x + self.norm(p + "norm2b", y)
        return x

    def streams(self, tokens: List[int]) -> List[torch.Tensor]:
        """The stream after the embedding and after every layer."""
        x = self.w["embed"][torch.tensor(tokens)]
        out = [x]
        for i in range(len(self.cfg["layers"])):
            x = self.layer(i, x)
            out.append(x)
        return out

    def logits(self, tokens: List[int]) -> torch.Tensor:
        return self.norm("final.norm", self.streams(tokens)[-1]) @ self.w["embed"].T


# ---------------------------------------------------------------- random models for the tests
def tensor_shapes(cfg: Dict) -> Dict[str, tuple]:
    """Name -> shape of every tensor of a model."""
    e, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, e)}

    def norm(name):
        out.update({name: (e,), name + ".b": (e,), name + ".alpha": ()})

    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        norm(p + "norm1")
        norm(p + "norm1b")
        m = layer["mixer"]
        q = p + "mix."
        if layer["type"] == "latent_attention":
            h, d, r, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
            out.update({q + "dq": (m["q_rank"], e), q + "dq.norm": (m["q_rank"],), q + "uq": (h * (d + r), m["q_rank"]),
                        q + "dkv": (m["kv_rank"] + r, e), q + "dkv.norm": (m["kv_rank"],), q + "uk": (h * d, m["kv_rank"]),
                        q + "uv": (h * dv, m["kv_rank"]), q + "o": (e, h * dv)})
        elif layer["type"] == "attention":
            nq, nk = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            out.update({q + "q": (nq, e), q + "k": (nk, e), q + "v": (m["kv_heads"] * m["vdim"], e), q + "q.norm": (nq,),
                        q + "k.norm": (nk,), q + "pb": (m["heads"],), q + "o": (e, m["heads"] * m["vdim"])})
        else:
            nq, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({q + "q": (nq, e), q + "k": (nq, e), q + "v": (nv, e), q + "g": (nv, e), q + "norm": (nv,), q + "o": (e, nv)})
        if layer.get("mlp") is not None:
            norm(p + "norm2")
            norm(p + "norm2b")
            ff, n = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"]["experts"]
            out.update({p + "mlp.router": (n, e), p + "mlp.router.b": (n,)})
            for x in range(n):
                out.update({f"{p}mlp.e{x}.gate": (ff, e), f"{p}mlp.e{x}.up": (ff, e), f"{p}mlp.e{x}.down": (e, ff)})
    return out


def random_lilevik_tensors(cfg: Dict, seed: int) -> Dict[str, torch.Tensor]:
    """Weights that bfloat16 holds exactly, so that the oracle and a model loaded from a bfloat16 file see the same numbers.
    Sizes are chosen so that every mechanism matters at tiny widths."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        base, last = name.rsplit(".", 1)[0], name.rsplit(".", 1)[-1]
        if last == "alpha":
            t = 0.5 + 0.4 * torch.rand(shape, generator=g)
        elif last == "b" and not base.endswith("router"):
            t = 0.2 * torch.randn(shape, generator=g)
        elif "norm" in last:
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif last == "pb":
            t = -2.0 + torch.randn(shape, generator=g)
        elif last == "b":
            t = torch.randn(shape, generator=g)
        elif name == "embed":
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) * (1.5 / math.sqrt(shape[-1]))
        out[name] = t.to(torch.bfloat16).to(F64)
    return out
