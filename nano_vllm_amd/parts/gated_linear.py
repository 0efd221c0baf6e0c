"""Mixer "gated_linear": linear attention whose state forgets by a decay per key channel that depends on the token, over a
state of fixed size per request (no denominator, no correction).

    q = h Wq^T * head_dim^-1/2,  k = h Wk^T     num_heads heads of head_dim;   v = h Wv^T: num_heads heads of v_head_dim
    a = sigmoid(z)^(1/tau),  z = (h Wa1^T) Wa2^T + b              per head and key channel
    S <- diag(a) S + k v^T;   o = S^T q                           per head, S [head_dim, v_head_dim]
    y = o / sqrt(mean(o^2) + eps) * w_norm * silu(h Wg^T)         per head; w_norm shared by the heads
    out = y Wo^T

Per request the layer keeps S in its state slot (FixedState), float32, zero at a request's start.  The decay from its
logits on, its logarithm and exponentials, the state, the read-out, the norm and the gate are float whatever the element
type.  The rank of the two-step projection (Wa1/Wa2) is the checkpoint's: its tensors' shapes decide it unless the parameters
name it.  The step's metadata is read on the device only, so single-token steps can be captured and replayed.
"""
from __future__ import annotations

from typing import Dict, Mapping

import torch

from .base import BuildContext, ParamDecl, Part, Source
from .registry import register_part
from .spec import FixedState


class GatedLinear(Part):
    """params: hidden_size, num_heads, head_dim, v_head_dim, tau, eps, decay_rank (None: the checkpoint's tensors decide;
    random weights then take head_dim / 4, at least 1), and the names of the checkpoint tensors (q_name, k_name, v_name,
    g_name, a1_name, a2_name, o_name, norm_name)."""

    replays_state_steps = True
    kernel_modules = ("memory",)

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        p = params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.dim = int(p["head_dim"])
        self.vdim = int(p.get("v_head_dim") or self.dim)
        self.tau = float(p["tau"])
        if not self.tau > 0:
            raise ValueError(f"gated_linear: tau {self.tau}")
        self.eps = float(p.get("eps", 1e-6))
        self.rank = None if p.get("decay_rank") is None else int(p["decay_rank"])
        self.names = {n: p.get(f"{n}_name", f"{n}_proj") for n in ("q", "k", "v", "g", "a1", "a2", "o")}
        self.norm_name = p.get("norm_name", "norm")
        self.rows = 2 * self.heads * (self.dim + self.vdim)

    def param_decls(self) -> Dict[str, ParamDecl]:
        n, qk, vv, h = self.names, self.heads * self.dim, self.heads * self.vdim, self.hidden
        rank, drawn = self.rank or -1, self.rank or max(1, self.dim // 4)
        return {
            "proj.weight": ParamDecl((self.rows, h), sources=tuple(
                Source(f"{n[name]}.weight", r, c) for name, r, c in (("q", 0, qk), ("k", qk, qk), ("v", 2 * qk, vv), ("g", 2 * qk + vv, vv)))),
            f"{n['a1']}.weight": ParamDecl((rank, h), default_shape=(drawn, h)),
            f"{n['a2']}.weight": ParamDecl((qk, rank), default_shape=(qk, drawn)),
            f"{n['a2']}.bias": ParamDecl((qk,), dtype="float32"),
            f"{self.norm_name}.weight": ParamDecl((self.vdim,), dtype="float32", init="norm"),
            f"{n['o']}.weight": ParamDecl((h, vv)),
        }

    def on_weights_loaded(self) -> None:
        # the decay's first step lies below q, k, v and the gate in one product (rows rounded up to whole vectors)
        w, n = self.weights, self.names
        a1, a2, proj = w[f"{n['a1']}.weight"], w[f"{n['a2']}.weight"], w["proj.weight"]
        if a1.shape[0] != a2.shape[1]:
            raise ValueError(f"gated_linear: the two steps of the decay's projection differ in rank ({tuple(a1.shape)} and {tuple(a2.shape)})")
        if proj.shape[0] == self.rows:
            pad = -(self.rows + a1.shape[0]) % 8
            w["proj.weight"] = torch.cat((proj, a1, proj.new_zeros((pad, self.hidden))), dim=0).contiguous()

    def cache_need(self):
        return FixedState({"s": ((self.heads, self.dim, self.vdim), "float32")})

    def forward(self, x, batch, cache):
        k, w, n = self.kernels, self.weights, self.names
        proj = k.linear(x, w["proj.weight"])
        y = k.gated_linear(proj, self.heads, self.dim, self.vdim, w[f"{n['a2']}.weight"], w[f"{n['a2']}.bias"], self.tau,
                           w[f"{self.norm_name}.weight"], self.eps, cache.state["s"], batch)
        return k.linear(y, w[f"{n['o']}.weight"], deferred=True)


register_part("mixer", "gated_linear", GatedLinear)
