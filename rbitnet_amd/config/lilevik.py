"""Typed configuration of the Lilevik decoder, read from config.json.

A decoder with a norm in front of and behind every sublayer: x <- x + norm1b(mixer(norm1(x))),
x <- x + norm2b(experts(norm2(x))); every norm of the model is tanh(alpha x) w + b, number by number, without statistics.
The order of layers is the file's; each has one of three mixers:
  "latent_attention"  causal softmax attention whose queries, keys and values go through latents; a head's key is a part made
                      from the cached latent beside a rotated part that all heads share (pairs 2i, 2i + 1);
  "attention"         grouped-query attention with norms over the whole of q and of k, a rotation of the head's first numbers
                      (pairs 2i, 2i + 1; wavelengths stretched by a ramp over the pairs, cosine and sine scaled), values divided
                      by their root mean square, keys limited to the query's chunk of `mask.size` positions, and weights that
                      are sigmoids of score plus a number per head, not normalised over the keys;
  "lightning"         linear attention on silu(q), silu(k), silu(v) with a constant decay per head, a norm over all heads together
                      and a sigmoid gate on the read-out;
and a mixture of experts (a bias on the router's logits, the `top` largest, the softmax over these alone as weights on the
experts' outputs), or no feed-forward.  The output matrix is the embedding's table.

Keys: architecture, vocab, width, norm.eps (of the RMS norms inside the mixers), layers: [{"type", "mixer": {...}, "mlp":
{"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}} or null}].

Tensor names: embed, final.norm(.b, .alpha), and per layer i under `l<i>.`: norm1, norm1b, norm2, norm2b (each with .b and
.alpha), mix.*, mlp.*.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..errors import ConfigError
from .spec import LayerSpec, ModelSpec, PartSpec
from .tigutar import _float, _int, _obj

MAX_POSITIONS = 1 << 20        # config.json gives no limit; this bounds a sequence where nothing else does
TYPES = ("latent_attention", "attention", "lightning")


def _rot(m: Dict[str, Any], where: str, limit: int) -> Optional[Dict[str, Any]]:
    """The mixer's rotation, checked; None where it has none (no `rot`, or no rotated numbers)."""
    if m.get("rot") is None:
        return None
    rot = _obj(m, "rot", where)
    dims = _int(rot, "dims", f"{where} rot", zero_ok=True)
    if dims % 2 != 0 or dims > limit:
        raise ConfigError(f"{where}: rot.dims must be even and at most {limit}, found {dims}")
    if dims == 0:
        return None
    if not _float(rot, "base", f"{where} rot") > 0:
        raise ConfigError(f"{where} rot: base must be positive")
    if rot.get("scaling") is not None:
        scaling = _obj(rot, "scaling", f"{where} rot")
        for key in ("factor", "original", "fast", "slow"):
            if not _float(scaling, key, f"{where} rot scaling") > 0:
                raise ConfigError(f"{where} rot scaling: {key} must be positive")
        if rot["base"] == 1:
            raise ConfigError(f"{where} rot: a scaling needs a base other than 1")
    return rot


@dataclass
class LilevikConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: List[Dict[str, Any]] = field(default_factory=list)
    max_positions: int = MAX_POSITIONS

    architecture = "Lilevik"

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "LilevikConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config: 'layers' must be a list with at least one layer")
        cfg = cls(vocab=_int(d, "vocab", "config"), width=_int(d, "width", "config"),
                  norm_eps=_float(_obj(d, "norm", "config"), "eps", "norm"), layers=copy.deepcopy(layers),
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
            if layer["type"] == "latent_attention":
                for key in ("heads", "dim", "vdim", "q_rank", "kv_rank"):
                    _int(m, key, where)
                _int(m, "rot_dim", where, zero_ok=True)
                _float(m, "scale", where)
                rot = _rot(m, where, m["rot_dim"])
                if (rot["dims"] if rot else 0) != m["rot_dim"]:
                    raise ConfigError(f"{where}: the rotated part has rot_dim = {m['rot_dim']} numbers and all of them are rotated, "
                                      f"found rot.dims = {rot['dims'] if rot else 0}")
            elif layer["type"] == "attention":
                for key in ("heads", "kv_heads", "dim", "vdim"):
                    _int(m, key, where)
                if m["heads"] % m["kv_heads"] != 0:
                    raise ConfigError(f"{where}: {m['heads']} heads cannot share {m['kv_heads']} key/value heads")
                _float(m, "scale", where)
                _rot(m, where, m["dim"])
                if m.get("mask") is not None:
                    _int(_obj(m, "mask", where), "size", f"{where} mask")
            else:
                for key in ("heads", "dim", "vdim"):
                    _int(m, key, where)
                decay = m.get("decay")
                if not isinstance(decay, list) or len(decay) != m["heads"]:
                    raise ConfigError(f"{where}: decay must list a number for each of the {m['heads']} heads, found {decay!r}")
                for n, _ in enumerate(decay):
                    _float({"decay": decay[n]}, "decay", where)
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
                raise ConfigError(f"{where}: mlp must be null or of kind 'moe', found {mlp!r}")
            _int(_obj(mlp, "expert", f"{where} mlp"), "ff", f"{where} expert")
            router = _obj(mlp, "router", f"{where} mlp")
            if _int(router, "top", f"{where} router") > _int(router, "experts", f"{where} router"):
                raise ConfigError(f"{where} router: top {router['top']} of {router['experts']} experts")

    def to_dict(self) -> Dict[str, Any]:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "layers": copy.deepcopy(self.layers)}
        if self.max_positions != MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out

    # ------------------------------------------------------------------ the spec
    def _position(self, rot: Optional[Dict[str, Any]]) -> PartSpec:
        if rot is None:
            return PartSpec("none", {"max_positions": self.max_positions})
        params = {"head_dim": rot["dims"], "theta": float(rot["base"]), "style": "interleaved", "max_positions": self.max_positions}
        if rot.get("scaling") is not None:
            params["scaling"] = dict({k: float(rot["scaling"][k]) for k in ("factor", "original", "fast", "slow")}, rope_type="yarn")
        return PartSpec("rope", params)

    def _mixer(self, kind: str, m: Dict[str, Any], where: str) -> PartSpec:
        eps = self.norm_eps
        if kind == "latent_attention":
            rot = _rot(m, where, m["rot_dim"])
            return PartSpec("latent_attention", {
                "heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"], "q_rank": m["q_rank"], "kv_rank": m["kv_rank"],
                "scale": m["scale"], "eps": eps, "rot_dim": m["rot_dim"], "position": self._position(rot) if rot else None,
                "sink": False, "head_gate": False})
        if kind == "attention":
            mask = m.get("mask")
            return PartSpec("attention", {
                "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"], "value_dim": m["vdim"],
                "scale": m["scale"], "window": None, "chunk": None if mask is None else mask["size"],
                "qk_norm": {"eps": eps, "weight": True, "over": "projection"}, "value_norm": eps, "weights": "sigmoid",
                "position": self._position(_rot(m, where, m["dim"])),
                "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "score_bias": "pb"}})
        return PartSpec("lightning", {"heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"], "decay": list(m["decay"]), "eps": eps})

    def to_spec(self) -> ModelSpec:
        def norm() -> PartSpec:
            return PartSpec("tanh", {"size": self.width, "names": {"weight": "", "bias": "b", "alpha": "alpha"}})
        layers = []
        for i, layer in enumerate(self.layers):
            mlp = layer.get("mlp")
            ff = None if mlp is None else PartSpec("routed_experts", {
                "experts": mlp["router"]["experts"], "top": mlp["router"]["top"], "intermediate_size": mlp["expert"]["ff"],
                "limit": None, "score": "chosen", "bias": True, "weight_on": "output"})
            params = {"norm1b": norm()}
            if ff is not None:
                params["norm2b"] = norm()
            layers.append(LayerSpec(prefix=f"l{i}", block="sandwich", mixer=self._mixer(layer["type"], layer["mixer"], f"layer {i}"),
                                    feed_forward=ff, norm1=norm(), norm2=None if ff is None else norm(),
                                    segments={"norm1": "norm1", "mixer": "mix", "norm1b": "norm1b", "norm2": "norm2",
                                              "feed_forward": "mlp", "norm2b": "norm2b"}, params=params))
        return ModelSpec(
            architecture=self.architecture, hidden_size=self.width, vocab_size=self.vocab, max_positions=self.max_positions,
            layers=layers, embedding=PartSpec("table", {"name": "embed", "vocab_size": self.vocab}),
            head=PartSpec("linear", {"norm": norm(), "norm_name": "final.norm", "name": None, "vocab_size": self.vocab}))
