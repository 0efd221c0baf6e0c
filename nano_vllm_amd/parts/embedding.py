"""Token embedding and output head: the two ends of the model, parts like the others.

An embedding kind gives `forward(ids int32 [T]) -> [T, hidden]` and keeps its table in
`weights["weight"]` (one with `reads_batch = True` gives `forward(ids, batch, cache)`, cache being the LayerCache of what its
`cache_need()` asks for, or None); a model that adds the embedding again later asks it for `second_copy(h)`, what it gave in a
tensor of its own; a head kind gives `forward(x [R, hidden]) -> float32 [R, vocab]` and an
attribute `tied`: when true it declares no tensor of its own and the model hands it the
embedding's table as `weights["weight"]`.  Both are built with the model's `vocab_size` and
`hidden_size` added to their parameters.
"""
from __future__ import annotations

from typing import Mapping

from .base import BuildContext, ParamDecl, Part
from .registry import register_part
from .spec import FixedState


class TokenEmbedding(Part):
    """weight [vocab, hidden]; rows are gathered by token id (embed_head.py:24,38).  With the
    parameter `scale` the rows are multiplied by that constant in float and leave as float32: the
    start of a residual stream that is kept in float32."""

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        self.vocab, self.hidden = int(params["vocab_size"]), int(params["hidden_size"])
        scale = params.get("scale")
        self.scale = None if scale is None else float(scale)

    def param_decls(self):
        return {"weight": ParamDecl((self.vocab, self.hidden))}

    def second_copy(self, x):
        return self.kernels.copy_rows(x)

    def forward(self, ids):
        if self.scale is not None:
            return self.kernels.embedding_scaled(self.weights["weight"], ids, self.scale)
        return self.kernels.embedding(self.weights["weight"], ids)


class SummedEmbedding(Part):
    """The start of a float32 residual stream as a sum of learned rows, every sum in float:
        x = weight[token]  +  bigram[row]  +  positions[p]
    bigram: a second table with row (before * mul_prev + token * mul_cur) mod buckets, `before` the token before this
    one in its sequence; a sequence's first token has the table's last row, number `buckets`.  The token before a
    portion's first one is kept per request (FixedState), so that a step reads its own tokens only; it is read and
    written on the device.  positions: a table of that many rows, one per position from 0 on; both are optional."""

    reads_batch = True
    replays_state_steps = True

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        self.vocab, self.hidden = int(params["vocab_size"]), int(params["hidden_size"])
        b = params.get("bigram")
        self.bigram = None if b is None else (int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"]))
        if self.bigram is not None and (self.bigram[0] <= 0 or min(self.bigram) < 0):
            raise ValueError(f"summed_embedding: bigram {b!r}: positive buckets and factors of zero or more are needed")
        self.positions = int(params.get("positions") or 0)

    def param_decls(self):
        d = {"weight": ParamDecl((self.vocab, self.hidden))}
        if self.bigram is not None:
            d["bigram.weight"] = ParamDecl((self.bigram[0] + 1, self.hidden))
        if self.positions:
            d["positions.weight"] = ParamDecl((self.positions, self.hidden))
        return d

    def cache_need(self):
        return None if self.bigram is None else FixedState({"before": ((1,), "int32")})

    def forward(self, ids, batch, cache):
        w = self.weights
        return self.kernels.summed_embedding(w["weight"], ids, w.get("bigram.weight"), self.bigram, w.get("positions.weight"),
                                             None if cache is None else cache.state["before"], batch)

    def second_copy(self, x):
        return self.kernels.copy_rows(x)


class OutputHead(Part):
    """logits = x W^T in float32, W [vocab, hidden] (embed_head.py:61); tied: W is the
    embedding's storage and the checkpoint holds no tensor for it (qwen3.py:202-203).  With the
    parameter logit_scale the logits are multiplied by that constant, in float; with softcap they are capped smoothly,
    softcap * tanh(logits / softcap), in float."""

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        self.vocab, self.hidden = int(params["vocab_size"]), int(params["hidden_size"])
        self.tied = bool(params.get("tied", False))
        self.logit_scale = float(params.get("logit_scale", 1.0))
        cap = params.get("softcap")
        self.softcap = None if cap is None else float(cap)
        if self.softcap is not None and not self.softcap > 0:
            raise ValueError(f"output_head: a softcap of {self.softcap}")

    def param_decls(self):
        return {} if self.tied else {"weight": ParamDecl((self.vocab, self.hidden))}

    def forward(self, x):
        logits = self.kernels.linear(x, self.weights["weight"], out_float32=True)
        if self.logit_scale != 1.0:
            self.kernels.scale_(logits, self.logit_scale)
        if self.softcap is not None:
            self.kernels.softcap_(logits, self.softcap)
        return logits


register_part("embedding", "token_embedding", TokenEmbedding)
register_part("embedding", "summed_embedding", SummedEmbedding)
register_part("head", "output_head", OutputHead)
