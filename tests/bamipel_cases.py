"""Shared by the Bamipel tests on the CPU stand-ins and on the GPU: small configurations, model folders whose
weights are made so that a fault shows, and comparisons with the plain implementation (tests/plain_bamipel.py)."""
from __future__ import annotations

import os
import tempfile
from types import SimpleNamespace
from typing import Dict, List

import torch
from safetensors.torch import load_file, save_file

from nano_vllm_amd.config import BamipelConfig
from nano_vllm_amd.config import BamipelLayer as Layer
from nano_vllm_amd.config import HeadDeltaConfig as Delta
from nano_vllm_amd.config import HeadGateAttentionConfig as Att
from nano_vllm_amd.config import QueryLatentAttentionConfig as Lat
from nano_vllm_amd.config import WaveScalingConfig as Wave
from nano_vllm_amd.weights import write_random_model

import plain_bamipel as plain
from pemuvik_cases import errors, err, fill_cache, paged_batch      # noqa: F401  (nothing in them is one design's)

_lat_a = Lat(heads=3, dim=10, rot_dim=6, vdim=14, q_rank=18, kv_rank=20, scale=0.35, window=10, rot_base=50.0)
_att_a = Att(heads=4, kv_heads=2, dim=12, vdim=16, scale=0.4, rot_dims=8, rot_base=100.0, rot_scaling=Wave(4.0, 1.0, 4.0, 64.0))
_del_a = Delta(heads=4, kv_heads=2, dim=12, vdim=8, conv=3)
_lat_c = Lat(heads=1, dim=4, rot_dim=2, vdim=6, q_rank=3, kv_rank=5, scale=0.6, window=1, rot_base=10.0)
_del_e = Delta(heads=4, kv_heads=2, dim=48, vdim=40, conv=4)
_lat_e = Lat(heads=5, dim=48, rot_dim=32, vdim=56, q_rank=72, kv_rank=96, scale=0.12, window=150, rot_base=2e4)

# Five configurations.  Together: latent windows smaller and larger than a page and no multiple of it, a window of one
# position, one longer than every prompt and none at all; query latents smaller and larger than the key latents; 1, 2, 3
# and H query heads per key/value head; values larger, smaller and as large as keys; rotation of a part of a head, of all
# of it and none, with and without scaled frequencies; delta layers first, last and in a row with 1, 2 and H query/key
# heads and convolutions of 1 to 5 taps; layers of every kind that run another layer's tensors again (one before its
# owner); layers without a feed-forward; sizes that are no multiples of 8.
CONFIGS: Dict[str, dict] = {
    "a": dict(cfg=BamipelConfig(vocab=200, width=48, eps=1e-5, layers=(
        Layer("latent_attention", _lat_a, 40, 0),
        Layer("delta", _del_a, 36, 1),
        Layer("latent_attention", _lat_a, 40, 0),
        Layer("attention", _att_a, None, 3),
        Layer("delta", _del_a, 36, 1),
        Layer("attention", _att_a, None, 3),
        Layer("latent_attention", Lat(2, 8, 4, 10, 30, 12, 0.3, window=21, rot_base=1e4), None, 6))), page=8, seed=61),
    # sizes of the matrix cores' kind
    "b": dict(cfg=BamipelConfig(vocab=512, width=128, eps=1e-6, layers=(
        Layer("delta", Delta(heads=4, kv_heads=2, dim=64, vdim=64, conv=4), 192, 0),
        Layer("latent_attention", Lat(8, 32, 16, 32, 64, 64, 0.2, window=48, rot_base=1e4), 192, 1),
        Layer("attention", Att(8, 2, 64, 64, 0.125, rot_dims=64, rot_base=2e5, rot_scaling=Wave(8.0, 1.0, 4.0, 32.0)), 192, 2),
        Layer("latent_attention", Lat(8, 32, 16, 32, 64, 64, 0.2, window=48, rot_base=1e4), 192, 1))), page=32, seed=62),
    # ones and equal values
    "c": dict(cfg=BamipelConfig(vocab=97, width=20, eps=1e-6, layers=(
        Layer("attention", Att(3, 1, 6, 10, 0.5, rot_dims=2, rot_base=300.0), 9, 1),
        Layer("attention", Att(3, 1, 6, 10, 0.5, rot_dims=2, rot_base=300.0), 9, 1),
        Layer("latent_attention", _lat_c, 8, 2),
        Layer("delta", Delta(1, 1, 4, 4, 1), None, 3),
        Layer("delta", Delta(3, 1, 5, 7, 5), 11, 4),
        Layer("latent_attention", Lat(2, 6, 2, 4, 8, 4, 0.5, window=4096, rot_base=300.0), 6, 5),
        Layer("attention", Att(1, 1, 8, 8, 0.35, rot_dims=0), 6, 6))), page=4, seed=63),
    "d": dict(cfg=BamipelConfig(vocab=333, width=72, eps=1e-6, layers=(
        Layer("delta", Delta(6, 6, 10, 14, 2), 100, 0),
        Layer("latent_attention", Lat(6, 12, 8, 10, 24, 40, 0.3, window=19, rot_base=1e6), 50, 1),
        Layer("attention", Att(6, 3, 24, 16, 0.3, rot_dims=24, rot_base=1e6, rot_scaling=Wave(2.0, 2.0, 2.0, 40.0)), 50, 2),
        Layer("latent_attention", Lat(4, 16, 6, 20, 16, 16, 0.3, window=None, rot_base=500.0), 50, 3),
        Layer("delta", Delta(6, 6, 10, 14, 2), 100, 0))), page=16, seed=64),
    # a larger one for long prompts: windows over several pages, key rows of exactly 128 entries and of more
    "e": dict(cfg=BamipelConfig(vocab=384, width=192, eps=1e-5, layers=(
        Layer("latent_attention", _lat_e, 256, 0),
        Layer("delta", _del_e, 256, 1),
        Layer("attention", Att(4, 4, 64, 64, 0.125, rot_dims=32, rot_base=2e4, rot_scaling=Wave(4.0, 1.0, 4.0, 256.0)), 256, 2),
        Layer("delta", _del_e, 256, 1),
        Layer("latent_attention", Lat(3, 64, 16, 32, 48, 176, 0.1, window=70, rot_base=1e5), 256, 4),
        Layer("latent_attention", _lat_e, 256, 0))), page=64, seed=65),
}

_folders: Dict[str, str] = {}
_tmp = None


def stretch(tensors: Dict[str, torch.Tensor], seed: int, sharp: bool = True) -> Dict[str, torch.Tensor]:
    """Random weights of N(0, std) hide faults: norms at one, gates at a half, decays that all lie together, scores too
    flat for a lost key to be missed.  This makes them of a size that shows.  sharp: also peaked scores, which the
    float32 tests want and which multiply bfloat16's rounding."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for k, t in tensors.items():
        f = t.float()
        draw = lambda: torch.randn(f.shape, generator=gen)
        if "norm" in k.rsplit(".", 1)[-1]:
            f = 1.0 + 0.4 * draw()
        elif k.endswith(".conv"):
            f = draw() * 0.6
        elif k.endswith(".dt_bias"):
            f = draw() - 0.5
        elif k.endswith(".A_log"):
            f = torch.log(0.03 + 0.6 * torch.rand(f.shape, generator=gen))
        elif k.endswith(".mix.g") or k.endswith(".mix.b") or k.endswith(".mix.a"):
            f = f * 3.0
        elif sharp and (k.endswith(".mix.uq") or k.endswith(".mix.dkv") or k.endswith(".mix.uk")):
            f = f * 2.5
        elif k == "embed":
            f = f * 5.0
        out[k] = f.to(t.dtype).contiguous()
    return out


def model_folder(name: str, dtype: str = "float32") -> str:
    global _tmp
    key = f"{name}-{dtype}"
    if key not in _folders:
        if _tmp is None:
            _tmp = tempfile.TemporaryDirectory(prefix="nva-bamipel-")
        c = CONFIGS[name]
        path = os.path.join(_tmp.name, key)
        write_random_model(path, c["cfg"], seed=c["seed"], std=0.1, dtype=dtype)
        file = os.path.join(path, "model.safetensors")
        save_file(stretch(load_file(file), c["seed"], sharp=dtype == "float32"), file, metadata={"format": "pt"})
        _folders[key] = path
    return _folders[key]


_plain_cache: Dict[str, tuple] = {}


def plain_model(folder: str):
    if folder not in _plain_cache:
        _plain_cache[folder] = plain.read_folder(folder, torch.float64)
    return _plain_cache[folder]


def plain_logits(folder: str, tokens: List[int]) -> torch.Tensor:
    cfg, w = plain_model(folder)
    return plain.forward(cfg, w, list(tokens)).float()


# ------------------------------------------------------------------------------ a delta-rule layer by itself
def delta_weights(shape, seed, dtype, slow=None):
    heads, kv_heads, dim, vdim, taps = shape
    g = torch.Generator().manual_seed(seed)
    C = 2 * kv_heads * dim + heads * vdim
    w = {"conv": (torch.randn((C, taps), generator=g) * 0.6).to(dtype), "dt_bias": torch.randn(heads, generator=g) - 0.5,
         "A_log": torch.log(0.02 + 1.5 * torch.rand(heads, generator=g)), "norm": 1 + 0.4 * torch.randn(vdim, generator=g)}
    if slow is not None:
        w["A_log"][slow] = -14.0           # a head that forgets next to nothing
    return w


def delta_inputs(shape, T, seed, dtype):
    """(projections [q | k | v | gate], rates [b | a])"""
    heads, kv_heads, dim, vdim, taps = shape
    g = torch.Generator().manual_seed(seed)
    C = 2 * kv_heads * dim + heads * vdim
    return ((torch.randn((T, C + heads * vdim), generator=g) * 1.5).to(dtype), torch.randn((T, 2 * heads), generator=g) * 1.5)


def plain_delta(shape, w, inputs, eps):
    heads, kv_heads, dim, vdim, taps = shape
    proj, rates = (t.double() for t in inputs)
    qk, vv = kv_heads * dim, heads * vdim
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim}
    conv = w["conv"].double()
    weights = {"q.conv": conv[:qk], "k.conv": conv[qk:2 * qk], "v.conv": conv[2 * qk:], "dt_bias": w["dt_bias"].double(),
               "A_log": w["A_log"].double(), "norm": w["norm"].double()}
    return plain.delta_of_projections(proj[:, :qk], proj[:, qk:2 * qk], proj[:, 2 * qk:2 * qk + vv], proj[:, 2 * qk + vv:],
                                      rates[:, :heads], rates[:, heads:], m, weights, "", eps)


def state_batch(dev, q_lens, starts, slots):
    token_seq = [s for s, n in enumerate(q_lens) for _ in range(n)]
    return SimpleNamespace(
        num_seqs=len(q_lens), q_lens=list(q_lens), starts=list(starts),
        num_decode=next((i for i, n in enumerate(q_lens) if n != 1), len(q_lens)),
        token_seq=torch.tensor(token_seq, dtype=torch.int32, device=dev),
        positions=torch.tensor([p for s, n in zip(starts, q_lens) for p in range(s, s + n)], dtype=torch.int32, device=dev),
        cu_seqlens_q=torch.tensor([0] + list(torch.tensor(q_lens).cumsum(0)), dtype=torch.int32, device=dev),
        seq_starts=torch.tensor(starts, dtype=torch.int32, device=dev),
        state_slots=torch.tensor(slots, dtype=torch.int32, device=dev))


def new_states(dev, slots, shape, fill=float("nan")):
    heads, kv_heads, dim, vdim, taps = shape
    C = 2 * kv_heads * dim + heads * vdim
    return (torch.full((slots, C, taps - 1), fill, dtype=torch.float32, device=dev),
            torch.full((slots, heads, dim, vdim), fill, dtype=torch.float32, device=dev))


def run_delta(k, dev, shape, w, inputs, eps, states, q_lens, starts, slots):
    heads, kv_heads, dim, vdim, taps = shape
    proj, rates = inputs
    out = k.head_delta(proj.to(dev), rates.to(dev).contiguous(), heads, kv_heads, dim, vdim, taps, w["conv"].to(dev),
                       w["dt_bias"].to(dev), w["A_log"].to(dev), w["norm"].to(dev), eps, states[0], states[1],
                       state_batch(dev, q_lens, starts, slots))
    k.check_faults()
    return out
