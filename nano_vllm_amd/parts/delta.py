"""Mixer "delta": the gated delta rule with one decay per head, over a state of fixed size per request (the
rule of "channel_delta" with a decay that all key channels of a head share, and a silu gate).

    q = h Wq^T, k = h Wk^T             kv_heads heads of head_dim;  v = h Wv^T: num_heads heads of v_head_dim
    q, k, v <- silu(causal convolution over the last `taps` tokens, per channel, no bias)
    q <- q / sqrt(sum(q^2) + 1e-6) * head_dim^-1/2,  k <- k / sqrt(sum(k^2) + 1e-6)         per head
    beta = sigmoid(h Wb^T),  a = exp(-exp(A_log) * softplus(h Wa^T + dt_bias))              one number per head each
    per head, with its query/key head floor(head / (num_heads / kv_heads)):
        S <- a S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q                     S [head_dim, v_head_dim]
    y = o / sqrt(mean(o^2) + eps) * w_norm * silu(h Wg^T)                                   per head; w_norm shared by the heads
    out = y Wo^T

Per request the layer keeps S and the last taps - 1 inputs of the three convolutions in its state slot
(FixedState), both float32, zero at a request's start.  Everything after the projections is float whatever the
element type, and the narrow projections of beta and the decay give float results.  The step's metadata is read on
the device only, so single-token steps can be captured and replayed.
"""
from __future__ import annotations

from typing import Dict, Mapping

from .base import BuildContext, ParamDecl, Part, Source
from .registry import register_part
from .spec import FixedState


class HeadDelta(Part):
    """params: hidden_size, num_heads, num_kv_heads, head_dim, v_head_dim, conv_taps, eps, and the names of the
    checkpoint tensors (q_name, k_name, v_name, b_name, a_name, g_name, o_name, norm_name, conv_suffix, dt_bias_name,
    a_log_name)."""

    replays_state_steps = True
    kernel_modules = ("delta",)

    def __init__(self, params: Mapping, build: BuildContext):
        super().__init__(params, build)
        p = params
        self.hidden = int(p["hidden_size"])
        self.heads = int(p["num_heads"])
        self.kv_heads = int(p.get("num_kv_heads") or self.heads)
        self.dim = int(p["head_dim"])
        self.vdim = int(p.get("v_head_dim") or self.dim)
        self.taps = int(p["conv_taps"])
        self.eps = float(p.get("eps", 1e-6))
        if self.heads % self.kv_heads:
            raise ValueError(f"delta: {self.heads} heads do not divide into {self.kv_heads} query/key heads")
        if self.taps < 1:
            raise ValueError("delta: a convolution has at least one tap (the token's own)")
        self.names = {n: p.get(f"{n}_name", f"{n}_proj") for n in ("q", "k", "v", "b", "a", "g", "o")}
        self.conv_suffix = p.get("conv_suffix", "conv")
        self.norm_name = p.get("norm_name", "norm")
        self.dt_bias_name = p.get("dt_bias_name", "dt_bias")
        self.a_log_name = p.get("a_log_name", "A_log")
        self.qk_channels = self.kv_heads * self.dim
        self.v_channels = self.heads * self.vdim
        self.conv_channels = 2 * self.qk_channels + self.v_channels

    def param_decls(self) -> Dict[str, ParamDecl]:
        n, qk, vv, h, H = self.names, self.qk_channels, self.v_channels, self.hidden, self.heads
        rows = ((n["q"], 0, qk), (n["k"], qk, qk), (n["v"], 2 * qk, vv))
        return {
            # q, k, v and the gate in one product; beta and the decay's input, which leave as float, in another
            "proj.weight": ParamDecl((self.conv_channels + vv, h), sources=tuple(
                Source(f"{name}.weight", r, c) for name, r, c in rows + ((n["g"], self.conv_channels, vv),))),
            "rates.weight": ParamDecl((2 * H, h), sources=(Source(f"{n['b']}.weight", 0, H), Source(f"{n['a']}.weight", H, H))),
            "conv.weight": ParamDecl((self.conv_channels, self.taps), sources=tuple(
                Source(f"{name}.{self.conv_suffix}.weight", r, c) for name, r, c in rows)),
            self.dt_bias_name: ParamDecl((H,), dtype="float32"),
            self.a_log_name: ParamDecl((H,), dtype="float32"),
            f"{self.norm_name}.weight": ParamDecl((self.vdim,), dtype="float32", init="norm"),
            f"{n['o']}.weight": ParamDecl((h, vv)),
        }

    def cache_need(self):
        return FixedState({"conv": ((self.conv_channels, self.taps - 1), "float32"),
                           "s": ((self.heads, self.dim, self.vdim), "float32")})

    def forward(self, x, batch, cache):
        k, w, n = self.kernels, self.weights, self.names
        proj = k.linear(x, w["proj.weight"])
        rates = k.linear(x, w["rates.weight"], out_float32=True, deferred=True)
        y = k.head_delta(proj, rates, self.heads, self.kv_heads, self.dim, self.vdim, self.taps, w["conv.weight"],
                         w[self.dt_bias_name], w[self.a_log_name], w[f"{self.norm_name}.weight"], self.eps,
                         cache.state["conv"], cache.state["s"], batch)
        return k.linear(y, w[f"{n['o']}.weight"], deferred=True)


register_part("mixer", "delta", HeadDelta)
