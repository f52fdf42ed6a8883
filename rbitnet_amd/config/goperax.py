"""Typed configuration of the Goperax decoder, read from config.json.

A decoder whose residual stream is kept in `streams` copies (hyper-connections): every sublayer reads a mixture of the copies
through an RMS norm, and all copies are then rebuilt from the old ones and the sublayer's result.  The stream starts as the
scaled embedding plus a fixed vector of sines and cosines of the position, and ends as the sum of the copies.  The order of layers
is the file's; a stretch of it may run several times in a row with the same weights (`loop`), each pass with a cache and
state of its own.  Each layer has one of two mixers:
  "mamba2"     a state-space mixer with a step size per token and head: a short convolution, the selective scan, a gate in front
               of a norm in equal parts;
  "attention"  grouped-query causal attention without positions whose values are its keys: scores capped by a tanh, the last
               `mask.size` keys, a softmax with one added to the denominator;
and a feed-forward with the squared relu: dense, a mixture of experts (the `top` largest of a softmax over all, divided by their
sum, as weights on the experts' outputs) with an expert that every token uses, or none.  The output matrix is the embedding's
table, without its scale.

Keys: architecture, vocab, width, streams, embedding.scale, norm.eps, loop: {"start", "stop", "times"} or null, layers: [{"type",
"mixer": {...}, "mlp": {"kind": "dense", "ff"} or {"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}, "shared": {"ff"}
or null} or null}].

Tensor names: embed, final.norm, and per layer i under `l<i>.`: norm1, norm2, hc1.{in,out,mix}, hc2.{in,out,mix}, mix.*, mlp.*.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..errors import ConfigError
from .spec import LayerSpec, ModelSpec, PartSpec
from .tigutar import _float, _int, _obj

MAX_POSITIONS = 1 << 20        # config.json gives no limit; this bounds a sequence where nothing else does
TYPES = ("mamba2", "attention")
WAVE_BASE = 10000.0            # of the sines and cosines added to the embedding


@dataclass
class GoperaxConfig:
    vocab: int
    width: int
    streams: int
    embedding_scale: float
    norm_eps: float
    layers: List[Dict[str, Any]] = field(default_factory=list)
    loop: Optional[Dict[str, int]] = None
    max_positions: int = MAX_POSITIONS

    architecture = "Goperax"

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "GoperaxConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config: 'layers' must be a list with at least one layer")
        loop = d.get("loop")
        cfg = cls(vocab=_int(d, "vocab", "config"), width=_int(d, "width", "config"), streams=_int(d, "streams", "config", 1),
                  embedding_scale=_float(_obj(d, "embedding", "config"), "scale", "embedding"),
                  norm_eps=_float(_obj(d, "norm", "config"), "eps", "norm"), layers=copy.deepcopy(layers),
                  loop=None if loop is None else dict(_obj(d, "loop", "config")),
                  max_positions=_int(d, "max_positions", "config", MAX_POSITIONS))
        cfg.check()
        return cfg

    # ------------------------------------------------------------------ checks
    def check(self) -> None:
        for i, layer in enumerate(self.layers):
            where = f"layer {i}"
            if not isinstance(layer, dict) or layer.get("type") not in TYPES:
                raise ConfigError(f"{where}: type must be one of {', '.join(TYPES)}, found "
                                  f"{layer.get('type') if isinstance(layer, dict) else layer!r}")
            m = _obj(layer, "mixer", where)
            if layer["type"] == "mamba2":
                for key in ("heads", "vdim", "state", "groups", "conv", "norm_groups"):
                    _int(m, key, where)
                if m["heads"] % m["groups"] != 0:
                    raise ConfigError(f"{where}: {m['heads']} heads cannot share {m['groups']} groups")
                if m["heads"] * m["vdim"] % m["norm_groups"] != 0:
                    raise ConfigError(f"{where}: {m['heads'] * m['vdim']} numbers cannot be normed in {m['norm_groups']} equal parts")
            else:
                for key in ("heads", "kv_heads", "dim"):
                    _int(m, key, where)
                if _int(m, "vdim", where, m["dim"]) != m["dim"]:
                    raise ConfigError(f"{where}: the values are the keys, so vdim must be dim = {m['dim']}, found {m['vdim']}")
                if m["heads"] % m["kv_heads"] != 0:
                    raise ConfigError(f"{where}: {m['heads']} heads cannot share {m['kv_heads']} key/value heads")
                _float(m, "scale", where)
                if m.get("softcap") is not None and not _float(m, "softcap", where) > 0:
                    raise ConfigError(f"{where}: softcap must be positive")
                if m.get("mask") is not None:
                    _int(_obj(m, "mask", where), "size", f"{where} mask")
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
                raise ConfigError(f"{where}: mlp must be null or of kind 'dense' or 'moe', found {mlp!r}")
            if mlp["kind"] == "dense":
                _int(mlp, "ff", f"{where} mlp")
                continue
            _int(_obj(mlp, "expert", f"{where} mlp"), "ff", f"{where} expert")
            router = _obj(mlp, "router", f"{where} mlp")
            if _int(router, "top", f"{where} router") > _int(router, "experts", f"{where} router"):
                raise ConfigError(f"{where} router: top {router['top']} of {router['experts']} experts")
            if mlp.get("shared") is not None:
                _int(_obj(mlp, "shared", f"{where} mlp"), "ff", f"{where} shared")
        if self.loop is not None:
            start, stop = (_int(self.loop, key, "loop", zero_ok=True) for key in ("start", "stop"))
            _int(self.loop, "times", "loop")
            if not start < stop <= len(self.layers):
                raise ConfigError(f"loop: layers {start} to {stop - 1} of {len(self.layers)} cannot be run over")

    def to_dict(self) -> Dict[str, Any]:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
               "embedding": {"scale": self.embedding_scale}, "norm": {"eps": self.norm_eps}, "layers": copy.deepcopy(self.layers)}
        if self.loop is not None:
            out["loop"] = dict(self.loop)
        if self.max_positions != MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out

    # ------------------------------------------------------------------ the spec
    def schedule(self) -> List[int]:
        """The layers in the order in which they run."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop = self.loop["start"], self.loop["stop"]
        return list(range(start)) + list(range(start, stop)) * self.loop["times"] + list(range(stop, n))

    def _mixer(self, kind: str, m: Dict[str, Any]) -> PartSpec:
        if kind == "mamba2":
            return PartSpec("state_space", dict({k: m[k] for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")}, eps=self.norm_eps))
        mask = m.get("mask")
        return PartSpec("attention", {
            "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"], "values": "keys", "scale": m["scale"],
            "softcap": m.get("softcap"), "window": None if mask is None else mask["size"], "sink": "one",
            "position": PartSpec("none", {"max_positions": self.max_positions}), "names": {"q": "q", "k": "k", "o": "o"}})

    @staticmethod
    def _feed_forward(mlp: Optional[Dict[str, Any]]) -> Optional[PartSpec]:
        if mlp is None:
            return None
        if mlp["kind"] == "dense":
            return PartSpec("dense_act", {"intermediate_size": mlp["ff"], "activation": "squared_relu"})
        shared = mlp.get("shared")
        # the softmax over all outputs divided by the chosen ones' sum is the softmax over the chosen logits alone
        return PartSpec("routed_experts", {
            "experts": mlp["router"]["experts"], "top": mlp["router"]["top"], "intermediate_size": mlp["expert"]["ff"], "limit": None,
            "score": "chosen", "weight_on": "output", "unit": "squared_relu",
            "shared": None if shared is None else {"intermediate_size": shared["ff"], "gate": False}})

    def to_spec(self) -> ModelSpec:
        def norm() -> PartSpec:
            return PartSpec("rmsnorm", {"size": self.width, "eps": self.norm_eps, "names": {"weight": ""}})
        layers, unused = [], []
        for i, layer in enumerate(self.layers):
            ff = self._feed_forward(layer.get("mlp"))
            if ff is None:                # a file may hold them all the same
                unused += [f"l{i}.norm2"] + [f"l{i}.hc2.{k}" for k in ("in", "out", "mix")]
            layers.append(LayerSpec(prefix=f"l{i}", block="hyper", mixer=self._mixer(layer["type"], layer["mixer"]), feed_forward=ff,
                                    norm1=norm(), norm2=None if ff is None else norm(),
                                    segments={"norm1": "norm1", "mixer": "mix", "norm2": "norm2", "feed_forward": "mlp"},
                                    params={"streams": self.streams, "scale": False}))
        return ModelSpec(
            architecture=self.architecture, hidden_size=self.width, vocab_size=self.vocab, max_positions=self.max_positions,
            layers=layers, schedule=self.schedule(), optional_tensors=unused,
            embedding=PartSpec("table", {"name": "embed", "vocab_size": self.vocab, "streams": self.streams,
                                         "scale": self.embedding_scale, "waves": WAVE_BASE}),
            head=PartSpec("linear", {"norm": norm(), "norm_name": "final.norm", "name": None, "vocab_size": self.vocab}))
