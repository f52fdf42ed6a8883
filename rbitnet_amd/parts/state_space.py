"""A state-space mixer with a step size per token and head (the selective scan of Mamba-2): per head a matrix S
[state, value size] in float32 that decays by the token's step size and takes in the token's own outer product.

Per token, with h the mixer's input, heads x vdim = inner and `groups` groups of key and query vectors that heads share
(head i reads group i // (heads // groups)):
    [z | x | k | q | t] = W_in h                 inner | inner | groups x state | groups x state | heads
    [x | k | q] <- silu(conv([x | k | q]) + b)   causal, per channel, `conv` taps
    dt = softplus(t + dt_bias)                   one number per head
    S <- exp(-exp(A_log) dt) S + dt k x^T;  y = S^T q + D x                 A_log and D one number per head
    y <- y * silu(z), each of `norm_groups` equal parts of it divided by its root mean square, times norm [inner];  out = Wo y
(k, q and t are often written B, C and dt.)

In float32: everything from the step sizes on, the recurrence, the gate and the norm.  Steps of many tokens a sequence run in
chunks on the matrix cores where the compute dtype is bfloat16 (the convolution then leaves bfloat16 numbers, which is what the
products take), steps of few tokens, float32 and other sizes one token after another.  The state lives in the cache's
per-slot storage (`view.states["scan"]`, [slots, heads, vdim, state], column by column), the convolution's last taps - 1 inputs
beside it (`view.states["conv"]`).

Parameters: heads, vdim, state, groups, conv (taps), norm_groups, eps, names (the tensors below the layer's prefix).
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..errors import ConfigError
from .base import BuildEnv, CacheRequest, Part, TensorSpec, register_mixer
from .linear import linear, linear_to_stream, pack_rows
from .short_conv import ACT_SILU, ShortConv

MAX_STATE = 512
CHUNKS_FROM = 24           # tokens of a step's longest piece from which chunks are worth their launches


class StateSpace(Part):
    graph_safe = True
    plan_safe = True
    leaves_terms = True

    NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "a_log": "A_log", "d": "D", "norm": "norm", "o": "o"}

    def __init__(self, params: Dict, env: BuildEnv):
        self.env = env
        self.heads, self.vdim = int(params["heads"]), int(params["vdim"])
        self.state, self.groups = int(params["state"]), int(params["groups"])
        self.norm_groups, self.eps = int(params["norm_groups"]), float(params["eps"])
        if min(self.heads, self.vdim, self.state, self.groups, self.norm_groups) <= 0 or self.state > MAX_STATE:
            raise ConfigError(f"state space: sizes must be positive, the state at most {MAX_STATE}")
        if self.heads % self.groups != 0:
            raise ConfigError(f"state space: {self.heads} heads cannot share {self.groups} groups")
        self.inner = self.heads * self.vdim
        if self.inner % self.norm_groups != 0:
            raise ConfigError(f"state space: {self.inner} numbers cannot be normed in {self.norm_groups} equal parts")
        self.names = dict(self.NAMES, **(params.get("names") or {}))
        self.hidden = env.hidden_size
        self.channels = self.inner + 2 * self.groups * self.state
        self.dt_col = self.inner + self.channels
        self.conv = ShortConv(self.channels, int(params["conv"]), env, residual=False, act=ACT_SILU)
        self.cache_from = None
        self.in_chunks = bool(env.dtype == torch.bfloat16 and env.lib is not None and not getattr(env, "generic_only", False)
                              and env.lib.selective_chunks_ok(self.state, self.vdim))

    # ------------------------------------------------------------------ tensors
    def tensor_specs(self) -> Dict[str, TensorSpec]:
        n, e = self.names, self.hidden
        gain = lambda *shape: TensorSpec(tuple(shape), role="gain", init="normal")
        return {n["in"]: TensorSpec((self.dt_col + self.heads, e)), n["conv"]: self.conv.tensor_spec(), n["conv_bias"]: gain(self.channels),
                n["dt_bias"]: gain(self.heads), n["a_log"]: gain(self.heads),
                n["d"]: TensorSpec((self.heads,), role="gain", init="ones_normal"),
                n["norm"]: TensorSpec((self.inner,), role="gain", init="ones_normal"), n["o"]: TensorSpec((e, self.inner))}

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        lib, allowed, n = self.env.lib, not getattr(self.env, "generic_only", False), self.names
        w = tensors[n["in"]]
        # rows up to a multiple of 16 (zeros), so that the product's kernels find whole tiles
        rows = (w.shape[0] + 15) // 16 * 16
        if rows != w.shape[0]:
            full = torch.zeros((rows, w.shape[1]), dtype=w.dtype, device=w.device)
            full[:w.shape[0]] = w
            w = full
        self.w_in = pack_rows(lib, [(w, 0, None, None)], rows, w.shape[1], w.dtype, w.device, allowed)
        self.conv.load(tensors[n["conv"]])
        self.conv_bias = tensors[n["conv_bias"]]
        self.dt_bias, self.a_log, self.d, self.norm = (tensors[n[k]] for k in ("dt_bias", "a_log", "d", "norm"))
        o = tensors[n["o"]]
        self.w_o = pack_rows(lib, [(o, 0, None, None)], o.shape[0], o.shape[1], o.dtype, o.device, allowed)

    def cache_requests(self) -> List[CacheRequest]:
        out = [CacheRequest("state", state_shape=(self.heads, self.vdim, self.state), state_init=0.0, name="scan")]
        conv = self.conv.cache_request("conv")
        return out + ([conv] if conv else [])

    def cache_request(self) -> Optional[CacheRequest]:
        return self.cache_requests()[0]

    # ------------------------------------------------------------------ forward
    def forward(self, h: torch.Tensor, ctx, view, stream: Optional[torch.Tensor] = None, next_norm=None) -> torch.Tensor:
        lib, t = self.env.lib, h.shape[0]
        proj = linear(lib, h, self.w_in, torch.float32)                       # [T, z | x | k | q | t]
        chunks = self.in_chunks and ctx.max_q_len >= CHUNKS_FROM
        xkq = self.conv.forward(proj, ctx, view.states.get("conv"), torch.bfloat16 if chunks else torch.float32, col0=self.inner,
                                bias_out=self.conv_bias)
        y = torch.empty((t, self.inner), dtype=torch.float32, device=h.device)
        scan = lib.selective_chunks if chunks else lib.selective_scan
        scan(xkq, self.state, self.groups, self.heads, self.vdim, proj, self.dt_col, self.dt_bias, self.a_log, self.d,
             view.states["scan"], ctx, y)
        yn = torch.empty((t, self.inner), dtype=self.env.dtype, device=h.device)
        lib.gate_rmsnorm_parts(y, self.norm, proj, 0, self.norm_groups, self.eps, yn)
        return linear_to_stream(lib, yn, self.w_o, None, next_norm)


register_mixer("state_space", StateSpace)
