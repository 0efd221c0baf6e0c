"""Bamipel as data: config.json -> typed configuration -> ModelSpec.

Every layer is the sandwich residual block on a float32 stream: an RMS norm before and one after each
sublayer, the normed output added to the stream.  The mixer is, entry by entry of the configuration's list, a
window attention through latents (queries through a normed latent of their own, keys and values through a normed
latent row and one rotated key part per token), a grouped attention (rotation whose frequencies may be scaled by
wavelength, query and key heads divided by their root mean square, every earlier key in sight) or the gated delta
rule with one decay per head (short convolutions, unit-norm queries and keys, a state of fixed size).  Both
attentions have an output gate of one number per head.  The feed-forward is W_d (max(W_u h, 0)^2), or absent.  The
head is untied.  An entry may run another entry's tensors again, with a cache or state of its own.

Checkpoint tensors: "embed", "head", "final.norm", and below "l<i>.": "norm1", "norm1b", "norm2", "norm2b",
"mix.<dq|uq|dkv|uk|uv|g|o>", "mix.<dq|dkv>.norm" (latents), "mix.<q|k|v|g|o>" (grouped attention),
"mix.<q|k|v|b|a|g|o>", "mix.<q|k|v>.conv", "mix.norm", "mix.dt_bias", "mix.A_log" (delta rule), "mlp.<up|down>": a
matrix is called by its part's name alone, which ModelSpec.checkpoint_names says.
"""
from __future__ import annotations

from dataclasses import asdict

from ..config.model_config import BamipelConfig, BamipelLayer
from ..config.registry import register_architecture
from ..parts.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

MAX_POSITION = 1 << 30          # the design names no longest sequence and keeps no table of positions


def _rotary_name(layer: BamipelLayer) -> str:
    m = layer.mixer
    if layer.kind == "latent_attention":
        return f"rotary-{m.rot_dim}-{m.rot_dim}-{m.rot_base!r}"
    s = m.rot_scaling
    return f"rotary-{m.dim}-{m.rot_dims}-{m.rot_base!r}" + ("" if s is None else f"-{s.factor!r}-{s.low!r}-{s.high!r}-{s.original!r}")


def _encodings(layer: BamipelLayer) -> dict:
    """The position encoding of a layer's mixer by its name, if it has one."""
    m = layer.mixer
    if layer.kind == "delta" or (layer.kind == "attention" and not m.rot_dims):
        return {}
    if layer.kind == "latent_attention":
        params = {"head_dim": m.rot_dim, "rotary_dim": m.rot_dim}
    else:
        params = {"head_dim": m.dim, "rotary_dim": m.rot_dims}
        if m.rot_scaling is not None:
            params["wave_scaling"] = asdict(m.rot_scaling)
    return {_rotary_name(layer): PartSpec("rotary_neox", {**params, "theta": m.rot_base, "max_position": MAX_POSITION})}


def _mixer(cfg: BamipelConfig, layer: BamipelLayer) -> PartSpec:
    m = layer.mixer
    if layer.kind == "latent_attention":
        return PartSpec("latent_attention", {
            "hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim, "v_head_dim": m.vdim,
            "q_rank": m.q_rank, "kv_rank": m.kv_rank, "eps": cfg.eps, "scale": m.scale, "window": m.window,
            "gate": "head_sigmoid", "position_encoding": _rotary_name(layer),
            "dq_name": "dq", "dq_norm_name": "dq.norm", "q_name": "uq", "dkv_name": "dkv", "dkv_norm_name": "dkv.norm",
            "uk_name": "uk", "uv_name": "uv", "g_name": "g", "o_name": "o"})
    if layer.kind == "attention":
        return PartSpec("attention", {
            "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
            "v_head_dim": m.vdim, "qk_norm": True, "qk_norm_scope": "head", "qk_norm_weight": False, "eps": cfg.eps,
            "bias": False, "position_encoding": _rotary_name(layer) if m.rot_dims else None, "step_rotation": True,
            "window": None, "scale": m.scale, "gate": "head_sigmoid",
            "q_name": "q", "k_name": "k", "v_name": "v", "g_name": "g", "o_name": "o"})
    return PartSpec("delta", {
        "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
        "v_head_dim": m.vdim, "conv_taps": m.conv, "eps": cfg.eps,
        **{f"{n}_name": n for n in ("q", "k", "v", "b", "a", "g", "o")},
        "conv_suffix": "conv", "norm_name": "norm", "dt_bias_name": "dt_bias", "a_log_name": "A_log"})


def build_spec(cfg: BamipelConfig) -> ModelSpec:
    norm = PartSpec("rms_norm", {"dim": cfg.width, "eps": cfg.eps})
    owners = [i for i, layer in enumerate(cfg.layers) if layer.weights_of == i]
    index = {i: n for n, i in enumerate(owners)}
    layers, encodings = [], {}
    for i in owners:
        layer = cfg.layers[i]
        encodings.update(_encodings(layer))
        parts = {"mixer_norm": norm, "mixer": _mixer(cfg, layer), "mixer_post_norm": norm}
        if layer.ff is not None:
            parts.update(feed_forward_norm=norm, feed_forward_post_norm=norm, feed_forward=PartSpec("mlp", {
                "hidden_size": cfg.width, "intermediate_size": layer.ff, "activation": "relu2",
                "up_name": "up", "down_name": "down"}))
        layers.append(LayerSpec(block=PartSpec("sandwich_residual"), parts=parts, name=f"l{i}",
                                names={"mixer_norm": "norm1", "mixer": "mix", "mixer_post_norm": "norm1b",
                                       "feed_forward_norm": "norm2", "feed_forward": "mlp",
                                       "feed_forward_post_norm": "norm2b"}))
    return ModelSpec(
        architecture=cfg.architecture, hidden_size=cfg.width, vocab_size=cfg.vocab, max_position=MAX_POSITION,
        dtype=cfg.dtype,
        # (a scale of one: the rows leave as the float32 stream)
        embedding=PartSpec("token_embedding", {"name": "embed", "scale": 1.0}),
        layers=tuple(layers),
        order=tuple(LayerRun(index[layer.weights_of]) for layer in cfg.layers),
        final_norm=PartSpec("rms_norm", {**norm.params, "name": "final.norm"}),
        head=PartSpec("output_head", {"name": "head", "tied": False}),
        position_encodings=encodings,
        eos_token_ids=cfg.eos_token_id or (),
        checkpoint_names=((".weight", ""), (".bias", ".b")),
    )


register_architecture("Bamipel", BamipelConfig.from_dict, build_spec, replace=True)
