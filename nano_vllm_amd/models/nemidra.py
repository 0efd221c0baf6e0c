"""Nemidra as data: config.json -> typed configuration -> ModelSpec.

The float32 residual stream starts as the sum of three embeddings: the token's, one by (token before, token), one by
position.  Every layer is the sandwich residual block with norms whose weights are stored around zero, followed by an
input of its own that every token brings from a table (the layer's part of the token's row).  The mixer is, entry by
entry of the configuration's list, a pair (a window attention with biases and no rotation, and a matrix memory with
exponential gates, added with a constant each) or a gated linear attention with a decay per key channel.  The
feed-forward is W_d gelu(W_u h), or a mixture of gated experts chosen and weighted by the softmax over all experts with a
shared expert behind a sigmoid gate, or absent.  Some layers run several times in a row with the same tensors, each
pass with a cache and state of its own, the embedding added to the stream before every pass but the first.  The head is
untied and its logits capped smoothly.

Checkpoint tensors: "embed", "bigram", "pos", "side.embed", "head", "final.norm", and below "l<i>.": "norm1", "norm1b",
"norm2", "norm2b", "mix.left.<q|k|v|o>" (+ ".b"), "mix.right.<q|k|v|g|o|norm>", "mix.right.<i|f>" (+ ".b"),
"mix.<q|k|v|g|o|norm|a1|a2>", "mix.a2.b" (gated linear attention), "mlp.<up|down>" (dense), "mlp.router",
"mlp.e<n>.<gate|up|down>", "mlp.shared.<gate|up|down|sg>", "side.<gate|proj|norm>".
"""
from __future__ import annotations

from ..config.model_config import NemidraConfig, NemidraLayer
from ..config.registry import register_architecture
from ..parts.spec import LayerRun, LayerSpec, ModelSpec, PartSpec


def _mixer(cfg: NemidraConfig, layer: NemidraLayer) -> PartSpec:
    m = layer.mixer
    if layer.kind == "gla":
        return PartSpec("gated_linear", {
            "hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "v_head_dim": m.vdim, "tau": m.tau,
            "eps": cfg.eps, "decay_rank": m.decay_rank, **{f"{n}_name": n for n in ("q", "k", "v", "g", "a1", "a2", "o")},
            "norm_name": "norm"})
    l, r = m.left, m.right
    left = PartSpec("attention", {
        "hidden_size": cfg.width, "num_heads": l.heads, "num_kv_heads": l.kv_heads, "head_dim": l.dim, "v_head_dim": l.vdim,
        "qk_norm": False, "bias": True, "o_bias": True, "eps": cfg.eps, "position_encoding": None, "window": l.window,
        "scale": l.scale, "q_name": "q", "k_name": "k", "v_name": "v", "o_name": "o"})
    right = PartSpec("matrix_memory", {
        "hidden_size": cfg.width, "num_heads": r.heads, "head_dim": r.dim, "v_head_dim": r.vdim, "gate_cap": r.gate_cap,
        "eps": cfg.eps, **{f"{n}_name": n for n in ("q", "k", "v", "g", "i", "f", "o")}, "norm_name": "norm"})
    return PartSpec("side_by_side", {
        "hidden_size": cfg.width, "eps": cfg.eps, "parts": {"left": left, "right": right},
        "names": {"left": "left", "right": "right"}, "combine": "scaled_sum", "scales": (m.left_scale, m.right_scale)})


def _feed_forward(cfg: NemidraConfig, layer: NemidraLayer) -> PartSpec:
    f = layer.mlp
    if isinstance(f, int):
        return PartSpec("mlp", {"hidden_size": cfg.width, "intermediate_size": f, "activation": "gelu", "up_name": "up",
                                "down_name": "down"})
    names = {"gate_name": "gate", "up_name": "up", "down_name": "down"}
    shared = None
    if f.shared_ff is not None:
        shared = PartSpec("swiglu", {"hidden_size": cfg.width, "intermediate_size": f.shared_ff, **names})
    return PartSpec("moe", {
        "hidden_size": cfg.width, "num_experts": f.experts, "top": f.top, "intermediate_size": f.ff, "scale": f.scale,
        "routing": "softmax_scores", "gated": True, "activation": "silu", "shared": shared, "shared_gate": shared is not None,
        "router_name": "router", "expert_name": "e{}", "shared_name": "shared", "shared_gate_name": "sg", **names})


def build_spec(cfg: NemidraConfig) -> ModelSpec:
    norm = PartSpec("rms_norm", {"dim": cfg.width, "eps": cfg.eps, "weight_offset": 1.0})
    plain_norm = PartSpec("rms_norm", {"dim": cfg.width, "eps": cfg.eps})
    tables = {}
    if cfg.side_dim is not None:
        tables["token_side"] = PartSpec("token_table", {"name": "side_table", "rows": cfg.vocab,
                                                        "width": len(cfg.layers) * cfg.side_dim})
    layers = []
    for i, layer in enumerate(cfg.layers):
        parts = {"mixer_norm": norm, "mixer": _mixer(cfg, layer), "mixer_post_norm": norm}
        if layer.mlp is not None:
            parts.update(feed_forward_norm=norm, feed_forward=_feed_forward(cfg, layer), feed_forward_post_norm=norm)
        if cfg.side_dim is not None:
            parts["token_side"] = PartSpec("token_side", {
                "hidden_size": cfg.width, "dim": cfg.side_dim, "offset": i * cfg.side_dim, "table": "token_side",
                "activation": "gelu_tanh", "norm": plain_norm, "gate_name": "gate", "proj_name": "proj", "norm_name": "norm"})
        layers.append(LayerSpec(block=PartSpec("sandwich_residual"), parts=parts, name=f"l{i}",
                                names={"mixer_norm": "norm1", "mixer": "mix", "mixer_post_norm": "norm1b",
                                       "feed_forward_norm": "norm2", "feed_forward": "mlp",
                                       "feed_forward_post_norm": "norm2b", "token_side": "side"}))
    start, stop, times = cfg.loop
    order = [LayerRun(i) for i in range(start)]
    for turn in range(times):
        order += [LayerRun(i, add_embedding=turn > 0 and i == start) for i in range(start, stop)]
    order += [LayerRun(i) for i in range(stop, len(layers))]
    embedding = {"name": "embed", "positions": cfg.max_positions}
    if cfg.bigram is not None:
        b = cfg.bigram
        embedding["bigram"] = {"buckets": b.buckets, "mul_prev": b.mul_prev, "mul_cur": b.mul_cur}
    return ModelSpec(
        architecture=cfg.architecture, hidden_size=cfg.width, vocab_size=cfg.vocab, max_position=cfg.max_positions,
        dtype=cfg.dtype, embedding=PartSpec("summed_embedding", embedding), layers=tuple(layers), order=tuple(order),
        final_norm=PartSpec("rms_norm", {**norm.params, "name": "final.norm"}),
        head=PartSpec("output_head", {"name": "head", "tied": False, "softcap": cfg.logit_softcap}),
        position_encodings={}, tables=tables, eos_token_ids=cfg.eos_token_id or (),
        checkpoint_names=(("embed.bigram.weight", "bigram"), ("embed.positions.weight", "pos"), ("side_table.weight", "side.embed"),
                          (".weight", ""), (".bias", ".b")),
    )


register_architecture("Nemidra", NemidraConfig.from_dict, build_spec, replace=True)
