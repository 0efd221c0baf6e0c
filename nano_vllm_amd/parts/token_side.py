"""What a layer takes from the step's tokens themselves.

Table "token_table": one row of `width` entries per token id, shared by the layers of a model, each of which reads a
part of the row.

"token_side": a sublayer that reads the residual stream x and the layer's part e = table[token, offset : offset + dim]:
    g = act(x Wg^T) * e;   y = g Wp^T
The norm through which y enters the stream is a part of it (`norm`; the block hands it on with y).  The activation is
float and g is rounded once.
"""
from __future__ import annotations

from typing import Dict, Mapping

from .base import BuildContext, ParamDecl, Part
from .registry import make_part, register_part


class TokenTable(Part):
    """params: rows, width."""

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        self.rows, self.width = int(params["rows"]), int(params["width"])

    def param_decls(self) -> Dict[str, ParamDecl]:
        return {"weight": ParamDecl((self.rows, self.width))}


class TokenSide(Part):
    """params: hidden_size, dim, offset (the first entry of the layer's part of a row), table (a name among the model's
    tables), activation (silu, relu, gelu_tanh, relu2, gelu), norm (a PartSpec), gate_name, proj_name, norm_name."""

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        self.hidden, self.dim, self.offset = int(params["hidden_size"]), int(params["dim"]), int(params["offset"])
        self.table = build.tables[params["table"]]
        if self.offset < 0 or self.offset + self.dim > self.table.width:
            raise ValueError(f"token_side: entries {self.offset} .. {self.offset + self.dim - 1} of a row of {self.table.width}")
        self.activation = params.get("activation", "gelu_tanh")
        self.gate_name, self.proj_name = params.get("gate_name", "gate"), params.get("proj_name", "proj")
        self.norm = make_part("norm", params["norm"], build)
        self.norm_name = params.get("norm_name", "norm")

    def children(self) -> Dict[str, Part]:
        return {self.norm_name: self.norm}

    def param_decls(self) -> Dict[str, ParamDecl]:
        return {f"{self.gate_name}.weight": ParamDecl((self.dim, self.hidden)),
                f"{self.proj_name}.weight": ParamDecl((self.hidden, self.dim))}

    def forward(self, x, ids):
        k, w = self.kernels, self.weights
        z = k.linear(x, w[f"{self.gate_name}.weight"], deferred=True)
        g = k.act_mul_rows(z, self.table.weights["weight"], ids, self.offset, self.activation)
        return k.linear(g, w[f"{self.proj_name}.weight"], deferred=True)


register_part("table", "token_table", TokenTable)
register_part("token_side", "token_side", TokenSide)
