"""Mixer "matrix_memory": a linear attention with an input gate and a forget gate per head that are exponentials of the
token's logits, kept in range by a running maximum, and with a denominator, over a state of fixed size per request.

    q = h Wq^T * head_dim^-1/2,  k = h Wk^T     num_heads heads of head_dim;   v = h Wv^T: num_heads heads of v_head_dim
    i = c tanh((h Wi^T + bi) / c),  f = logsigmoid(c tanh((h Wf^T + bf) / c))        one number per head, c = gate_cap
    m' = max(f + m, i);   S <- exp(f + m - m') S + exp(i - m') k v^T;   n <- exp(f + m - m') n + exp(i - m') k
    o = S^T q / (max(|n . q|, exp(-m')) + 1e-6)                  per head; m starts at 0, S and n at zero
    y = o / sqrt(mean(o^2) + eps) * w_norm * sigmoid(h Wg^T)     the norm per head, w_norm over all heads' channels
    out = y Wo^T

Per request the layer keeps S, n and m in its state slot (FixedState), float32.  The gates (their narrow product gives
float results), the state, the read-out, the norm and the output gate are float whatever the element type.  The step's
metadata is read on the device only, so single-token steps can be captured and replayed.
"""
from __future__ import annotations

from typing import Dict, Mapping

from .base import BuildContext, ParamDecl, Part, Source
from .registry import register_part
from .spec import FixedState


class MatrixMemory(Part):
    """params: hidden_size, num_heads, head_dim, v_head_dim, gate_cap, eps, and the names of the checkpoint tensors
    (q_name, k_name, v_name, g_name, i_name, f_name, o_name, norm_name)."""

    replays_state_steps = True
    kernel_modules = ("memory",)

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        p = params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.dim = int(p["head_dim"])
        self.vdim = int(p.get("v_head_dim") or self.dim)
        self.cap = float(p["gate_cap"])
        if not self.cap > 0:
            raise ValueError(f"matrix_memory: a gate cap of {self.cap}")
        self.eps = float(p.get("eps", 1e-6))
        self.names = {n: p.get(f"{n}_name", f"{n}_proj") for n in ("q", "k", "v", "g", "i", "f", "o")}
        self.norm_name = p.get("norm_name", "norm")

    def param_decls(self) -> Dict[str, ParamDecl]:
        n, qk, vv, h, H = self.names, self.heads * self.dim, self.heads * self.vdim, self.hidden, self.heads
        return {
            # q, k, v and the output gate in one product; the two gates' logits, which leave as float, in another
            "proj.weight": ParamDecl((2 * qk + 2 * vv, h), sources=tuple(
                Source(f"{n[name]}.weight", r, c) for name, r, c in (("q", 0, qk), ("k", qk, qk), ("v", 2 * qk, vv), ("g", 2 * qk + vv, vv)))),
            "gates.weight": ParamDecl((2 * H, h), sources=(Source(f"{n['i']}.weight", 0, H), Source(f"{n['f']}.weight", H, H))),
            "gates.bias": ParamDecl((2 * H,), dtype="float32", sources=(Source(f"{n['i']}.bias", 0, H), Source(f"{n['f']}.bias", H, H))),
            f"{self.norm_name}.weight": ParamDecl((vv,), dtype="float32", init="norm"),
            f"{n['o']}.weight": ParamDecl((h, vv)),
        }

    def cache_need(self):
        return FixedState({"s": ((self.heads, self.dim, self.vdim), "float32"), "n": ((self.heads, self.dim), "float32"),
                           "m": ((self.heads,), "float32")})

    def forward(self, x, batch, cache):
        k, w, n = self.kernels, self.weights, self.names
        proj = k.linear(x, w["proj.weight"])
        gates = k.linear(x, w["gates.weight"], out_float32=True, deferred=True)
        y = k.matrix_memory(proj, gates, w["gates.bias"], self.heads, self.dim, self.vdim, self.cap,
                            w[f"{self.norm_name}.weight"], self.eps, cache.state["s"], cache.state["n"], cache.state["m"], batch)
        return k.linear(y, w[f"{n['o']}.weight"], deferred=True)


register_part("mixer", "matrix_memory", MatrixMemory)
