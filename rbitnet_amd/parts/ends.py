"""The two ends of a model: what turns token ids into the residual stream, and what turns
the stream into logits.  Parts like the others: a kind in a registry, parameters, tensors of
their own, a forward; a model's forward is the embedding, the blocks in schedule order, the
head, and holds no stage of its own.  An architecture that scales its embeddings, or scales or
caps its logits, or computes them in another way, registers another kind.

Their tensors have no layer prefix: `tensor_specs` names them in full.

embedding "table" (crates/bitnet-core/src/llama/model.rs:229-232): x[t, :] = table[id[t], :].
    Parameters: name, vocab_size, streams (None: the stream is [T, E]; n: n equal copies [n, T, E], for
    blocks that keep the residual stream in several copies), scale (None, or c: the rows are multiplied by c),
    positions (None, or {"name": tensor, "max_positions": n}: a learned vector per absolute position [n, E], added
    to the scaled row as it is): x[t, :] = table[id[t], :] * c + positions[pos[t], :]; waves (None, or b: a fixed vector per
    absolute position p is added, whose numbers 2i and 2i + 1 are the sine and the cosine of p b^(-2i / E); with `scale` it also goes
    with several copies of the stream); norm (None, or a PartSpec of a norm
    that offers `add_normed`) with norm_name (its tensor): the stream starts as norm(row), and the first block also gets
    these rows in the compute dtype (forward then returns the stream and a `StreamCopy`).
    Interface of an embedding: tensor_specs() / load(tensors) / forward(ctx) -> float32 [T, E]
    (ctx.token_ids int32 [T]); `table` if a head may share it.

head "linear" (model.rs:309-315): logits = W norm(x), on the asked rows only; W is the
    embedding's table when the parameters name no matrix (tied).
    Parameters: norm (a PartSpec), norm_name, name (None: tied), vocab_size, softcap (None, or c:
    logits <- c tanh(logits / c)), logit_scale (None, or s: logits <- s logits, before a cap).  A stream in several
    copies is summed by the norm.
    Interface of a head: tensor_specs() / load(tensors, embedding) /
    forward(x, pending, rows, ctx) -> float32 [len(rows), V], where x is the stream, `pending`
    what the last block left to be added (see stream.py) and rows the packed rows asked for;
    first_norm (optional): the norm it begins with, for the last block.
    step_bytes(element_size) (optional, both ends): the bytes of its tensors that a step reads
    in full (default: all of them).
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..errors import ConfigError
from .base import BuildEnv, Part, TensorSpec, build_part, register_embedding, register_head
from .linear import linear, pack_rows
from .stream import StreamCopy, normed_for


class TableEmbedding(Part):

    def __init__(self, params: Dict, env: BuildEnv):
        self.env = env
        self.name = str(params["name"])
        self.vocab_size = int(params["vocab_size"])
        self.hidden = env.hidden_size
        self.streams = None if params.get("streams") is None else int(params["streams"])
        self.scale = None if params.get("scale") is None else float(params["scale"])
        pos = params.get("positions")
        self.pos_name = None if pos is None else str(pos["name"])
        self.max_positions = None if pos is None else int(pos["max_positions"])
        self.waves = None if params.get("waves") is None else float(params["waves"])
        if pos is not None and (self.streams is not None or self.waves is not None):
            raise ConfigError("an embedding with learned positions fills one copy of the stream, and has no waves")
        if self.waves is not None and not self.waves > 0:
            raise ConfigError(f"an embedding's waves need a positive base, found {self.waves}")
        self.inv = None
        if self.waves is not None and env.lib is not None:
            i = torch.arange((self.hidden + 1) // 2, dtype=torch.float64)
            self.inv = torch.pow(torch.tensor(self.waves, dtype=torch.float64), -2.0 * i / self.hidden).to(env.device)
        self.norm = None
        if params.get("norm") is not None:
            self.norm = build_part("norm", params["norm"], env)
            self.norm_name = str(params["norm_name"])
            if self.streams is not None or not hasattr(self.norm, "add_normed") or len(self.norm.tensor_specs()) != 1:
                raise ConfigError("a norm behind the embedding: one copy of the stream, and a norm of one tensor that can stand on an output")
        self.table: Optional[torch.Tensor] = None
        self.positions: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        out = {self.name: TensorSpec((self.vocab_size, self.hidden))}
        if self.pos_name is not None:
            out[self.pos_name] = TensorSpec((self.max_positions, self.hidden))
        if self.norm is not None:
            out[self.norm_name] = next(iter(self.norm.tensor_specs().values()))
        return out

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.table = tensors[self.name]
        if self.pos_name is not None:
            self.positions = tensors[self.pos_name]
        if self.norm is not None:
            self.norm.load({next(iter(self.norm.tensor_specs())): tensors[self.norm_name]})

    @property
    def graph_safe(self) -> bool:
        return self.norm is None or bool(getattr(self.norm, "graph_safe", False))

    @property
    def plan_safe(self) -> bool:
        return self.norm is None or bool(getattr(self.norm, "plan_safe", False))

    def step_bytes(self, element_size: int) -> int:
        return 0                      # the gather reads a few rows only

    def forward(self, ctx) -> torch.Tensor:
        if self.streams is not None:
            x = torch.empty((self.streams, ctx.n_tokens, self.hidden), dtype=torch.float32, device=self.table.device)
            if self.waves is not None or self.scale is not None:
                self.env.lib.embed_streams_waves(self.table, ctx.token_ids, 1.0 if self.scale is None else self.scale, self.inv,
                                                 ctx.tok_pos, x)
            else:
                self.env.lib.embed_streams(self.table, ctx.token_ids, x)
            return x
        x = torch.empty((ctx.n_tokens, self.hidden), dtype=torch.float32, device=self.table.device)
        if self.waves is not None:
            self.env.lib.embed_streams_waves(self.table, ctx.token_ids, 1.0 if self.scale is None else self.scale, self.inv,
                                             ctx.tok_pos, x.unsqueeze(0))
        elif self.scale is not None or self.positions is not None:
            self.env.lib.embed_scaled_pos(self.table, ctx.token_ids, 1.0 if self.scale is None else self.scale,
                                          self.positions, ctx.tok_pos, x)
        else:
            self.env.lib.embed_gather(self.table, ctx.token_ids, x)
        if self.norm is not None:
            rows = torch.empty((ctx.n_tokens, self.hidden), dtype=torch.float32, device=x.device)
            h = rows if self.env.dtype == torch.float32 else torch.empty_like(rows, dtype=self.env.dtype)
            self.norm.add_normed(rows, x, h_out=None if h is rows else h, assign=True)
            return rows, StreamCopy(h)
        return x


class LinearHead(Part):
    takes_gained_rows = True      # the output product takes what the last product left for the final norm

    def __init__(self, params: Dict, env: BuildEnv):
        self.env = env
        self.norm = build_part("norm", params["norm"], env)
        self.norm_name = str(params["norm_name"])
        self.name = params.get("name")
        self.vocab_size = int(params["vocab_size"])
        self.hidden = env.hidden_size
        self.softcap = None if params.get("softcap") is None else float(params["softcap"])
        if self.softcap is not None and not self.softcap > 0:
            raise ConfigError(f"a head's softcap must be positive, found {self.softcap}")
        self.logit_scale = None if params.get("logit_scale") is None else float(params["logit_scale"])
        self.weight = None

    @property
    def graph_safe(self) -> bool:
        return bool(getattr(self.norm, "graph_safe", False))

    @property
    def plan_safe(self) -> bool:
        return bool(getattr(self.norm, "plan_safe", False))

    @property
    def first_norm(self):
        return self.norm

    def _norm_names(self) -> Dict[str, str]:
        """full name -> the norm's own name of the tensor"""
        specs = self.norm.tensor_specs()
        if hasattr(self.norm, "tensor_names"):
            return self.norm.tensor_names(self.norm_name)
        if len(specs) == 1:
            return {self.norm_name: next(iter(specs))}
        base = self.norm_name.rsplit(".", 1)[0]
        return {f"{base}.{name}": name for name in specs}

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        own = self.norm.tensor_specs()
        out = {full: own[name] for full, name in self._norm_names().items()}
        if self.name is not None:
            out[str(self.name)] = TensorSpec((self.vocab_size, self.hidden))
        return out

    def load(self, tensors: Dict[str, torch.Tensor], embedding=None) -> None:
        self.norm.load({name: tensors[full] for full, name in self._norm_names().items()})
        if self.name is None:
            table = getattr(embedding, "table", None)
            if table is None or tuple(table.shape) != (self.vocab_size, self.hidden):
                raise ConfigError("a head without a matrix of its own needs an embedding whose table it can share")
            self.weight = table                 # tied: the table's rows are also read one by one, so it stays rows
            return
        w = tensors[str(self.name)]
        self.weight = pack_rows(self.env.lib, [(w, 0, None, None)], w.shape[0], w.shape[1], w.dtype, w.device,
                                not getattr(self.env, "generic_only", False))

    def step_bytes(self, element_size: int) -> int:
        gains = sum(4 * _numel(ts.shape) for ts in self.norm.tensor_specs().values())
        return gains + self.vocab_size * self.hidden * element_size        # tied or not, the matrix is read once

    def forward(self, x: torch.Tensor, pending, rows: torch.Tensor, ctx=None) -> torch.Tensor:
        xn = normed_for(self, self.norm, x, pending, rows)
        logits = linear(self.env.lib, xn, self.weight, torch.float32)
        if self.logit_scale is not None:
            self.env.lib.scale(logits, self.logit_scale)
        if self.softcap is not None:
            self.env.lib.tanh_cap(logits, self.softcap)
        return logits


def _numel(shape) -> int:
    n = 1
    for s in shape:
        n *= int(s)
    return n


register_embedding("table", TableEmbedding)
register_head("linear", LinearHead)
