"""Shared by the Nemidra tests on the CPU stand-ins and on the GPU: small configurations, model folders whose
weights are made so that a fault shows, and comparisons with the plain implementation (tests/plain_nemidra.py)."""
from __future__ import annotations

import os
import tempfile
from typing import Dict, List

import torch
from safetensors.torch import load_file, save_file

from nano_vllm_amd.config import BigramConfig as Bigram
from nano_vllm_amd.config import GatedLinearConfig as Gla
from nano_vllm_amd.config import MatrixMemoryConfig as Mem
from nano_vllm_amd.config import NemidraConfig
from nano_vllm_amd.config import NemidraLayer as Layer
from nano_vllm_amd.config import PairMixerConfig as Pair
from nano_vllm_amd.config import SoftmaxScoreExpertsConfig as Moe
from nano_vllm_amd.config import WindowAttentionConfig as Win
from nano_vllm_amd.weights import write_random_model

import plain_nemidra as plain
from bamipel_cases import state_batch                               # noqa: F401  (nothing in it is one design's)
from pemuvik_cases import errors, err, fill_cache, paged_batch      # noqa: F401

_pair_a = Pair(Win(4, 2, 12, 16, 0.4, window=10), Mem(3, 10, 14, 5.0), 0.7, 1.3)
_gla_a = Gla(3, 14, 10, 4.0, decay_rank=5)

# Five configurations.  Together: windows smaller and larger than a page and no multiple of it, of one position, longer than
# every prompt, and none; 1, 2, 3 and H query heads per key/value head; values larger, smaller and as large as keys, in all
# three mixers; loops over one layer, several, all, at the start, the middle and the end, once, twice and three times; dense,
# routed (with and without a shared expert, one expert, all experts) and absent feed-forwards; mixers first and last of either
# kind; sizes that are no multiples of 8; a bigram table of one bucket, factors of zero; scales of one and of zero.
CONFIGS: Dict[str, dict] = {
    "a": dict(cfg=NemidraConfig(vocab=200, width=48, eps=1e-5, max_positions=300, side_dim=10, bigram=Bigram(89, 7, 3), loop=(1, 3, 2),
                                logit_softcap=8.0, layers=(
        Layer("gla", _gla_a, 40),
        Layer("parallel", _pair_a, Moe(6, 2, 20, 1.5, shared_ff=28)),
        Layer("gla", _gla_a, Moe(5, 3, 16, 0.8)),
        Layer("parallel", Pair(Win(2, 1, 8, 8, 0.5, window=21), Mem(2, 16, 16, 12.0), 1.0, 0.5), None))), page=8, seed=71),
    # sizes of the matrix cores' kind
    "b": dict(cfg=NemidraConfig(vocab=512, width=128, eps=1e-6, max_positions=1024, side_dim=32, bigram=Bigram(251, 131, 17), loop=(0, 2, 2),
                                logit_softcap=20.0, layers=(
        Layer("parallel", Pair(Win(4, 2, 64, 64, 0.125, window=48), Mem(2, 64, 64, 15.0), 0.6, 0.9), Moe(8, 2, 64, 1.0, shared_ff=64)),
        Layer("gla", Gla(2, 64, 64, 16.0, decay_rank=16), 256))), page=32, seed=72),
    # ones, zeros and equal values
    "c": dict(cfg=NemidraConfig(vocab=97, width=20, eps=1e-6, max_positions=256, side_dim=1, bigram=Bigram(1, 0, 5), loop=(0, 1, 3),
                                logit_softcap=5.0, layers=(
        Layer("parallel", Pair(Win(1, 1, 4, 4, 0.5, window=1), Mem(1, 4, 4, 2.0), 1.0, 1.0), Moe(1, 1, 6, 1.0, shared_ff=1)),
        Layer("gla", Gla(1, 1, 1, 1.0, decay_rank=1), None),
        Layer("parallel", Pair(Win(3, 1, 6, 10, 0.5, window=4096), Mem(3, 5, 7, 1.0), 0.0, 1.0), 9),
        Layer("gla", Gla(3, 5, 7, 0.5, decay_rank=3), Moe(4, 4, 5, 2.0)))), page=4, seed=73),
    "d": dict(cfg=NemidraConfig(vocab=333, width=72, eps=1e-5, max_positions=512, side_dim=24, bigram=Bigram(1009, 31, 1), loop=(2, 4, 2),
                                logit_softcap=12.0, layers=(
        Layer("parallel", Pair(Win(6, 3, 24, 16, 0.25, window=19), Mem(4, 12, 20, 9.0), 1.2, 0.8), 100),
        Layer("parallel", Pair(Win(6, 6, 10, 14, 0.35, window=None), Mem(2, 20, 12, 9.0), 0.8, 1.2), Moe(12, 4, 24, 1.0, shared_ff=36)),
        Layer("gla", Gla(4, 18, 22, 8.0, decay_rank=8), Moe(12, 4, 24, 1.0, shared_ff=36)),
        Layer("gla", Gla(4, 18, 22, 8.0, decay_rank=8), 64))), page=16, seed=74),
    # a larger one for long prompts: windows over several pages, states of several tiles
    "e": dict(cfg=NemidraConfig(vocab=384, width=192, eps=1e-5, max_positions=1024, side_dim=48, bigram=Bigram(509, 37, 11), loop=(1, 2, 2),
                                logit_softcap=15.0, layers=(
        Layer("gla", Gla(2, 128, 96, 16.0, decay_rank=24), 256),
        Layer("parallel", Pair(Win(6, 2, 32, 32, 0.2, window=150), Mem(2, 96, 112, 10.0), 0.9, 0.7), Moe(8, 3, 64, 1.2, shared_ff=96)))),
        page=64, seed=75),
}

_folders: Dict[str, str] = {}
_tmp = None


def stretch(tensors: Dict[str, torch.Tensor], seed: int, sharp: bool = True) -> Dict[str, torch.Tensor]:
    """Random weights of N(0, std) hide faults: norms at one, gates at a half, decays that all lie together, scores too flat
    for a lost key to be missed.  This makes them of a size that shows.  sharp: also peaked scores and clear choices of
    experts, which the float32 tests want and which multiply bfloat16's rounding."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for k, t in tensors.items():
        f = t.float()
        draw = lambda: torch.randn(f.shape, generator=gen)
        last = k.rsplit(".", 1)[-1]
        if last.startswith("norm"):
            plain_weight = ".mix." in k or ".side." in k
            f = (1.0 if plain_weight else 0.0) + 0.4 * draw()
        elif k.endswith("right.f.b"):
            f = 2.0 + 2.0 * draw()
        elif k.endswith("right.i.b"):
            f = 1.5 * draw()
        elif k.endswith("a2.b"):
            f = 1.0 + 2.0 * draw()
        elif k.endswith(".b"):
            f = 0.3 * draw()
        elif k.endswith("right.i") or k.endswith("right.f") or k.endswith(".a2") or k.endswith(".mix.g") or k.endswith("right.g"):
            f = f * 3.0
        elif k.endswith(".router"):
            f = draw() * (0.6 if sharp else 0.15)
        elif k.endswith(".sg"):
            f = draw() * 0.4
        elif sharp and (k.endswith("left.q") or k.endswith("left.k")):
            f = f * 2.5
        elif k in ("embed", "bigram", "pos"):
            f = f * 5.0
        elif k == "side.embed":
            f = f * 10.0
        elif k == "head":
            f = f * 3.0
        out[k] = f.to(t.dtype).contiguous()
    return out


def model_folder(name: str, dtype: str = "float32") -> str:
    global _tmp
    key = f"{name}-{dtype}"
    if key not in _folders:
        if _tmp is None:
            _tmp = tempfile.TemporaryDirectory(prefix="nva-nemidra-")
        c = CONFIGS[name]
        path = os.path.join(_tmp.name, key)
        write_random_model(path, c["cfg"], seed=c["seed"], std=0.1, dtype=dtype)
        file = os.path.join(path, "model.safetensors")
        save_file(stretch(load_file(file), c["seed"], sharp=dtype == "float32"), file, metadata={"format": "pt"})
        _folders[key] = path
    return _folders[key]


_plain_cache: Dict[str, tuple] = {}
_logit_cache: Dict[tuple, torch.Tensor] = {}


def plain_model(folder: str):
    if folder not in _plain_cache:
        _plain_cache[folder] = plain.read_folder(folder, torch.float64)
    return _plain_cache[folder]


def plain_logits(folder: str, tokens: List[int]) -> torch.Tensor:
    key = (folder, tuple(tokens))
    if key not in _logit_cache:
        cfg, w = plain_model(folder)
        _logit_cache[key] = plain.forward(cfg, w, list(tokens)).float()
    return _logit_cache[key]


# ------------------------------------------------------------------------------ the two state layers by themselves
class LinearRule:
    """A gated linear attention: shape (heads, dim, vdim, rank, tau)."""
    def __init__(self, shape, seed, dtype, forget=None):
        self.heads, self.dim, self.vdim, self.rank, self.tau = shape
        g = torch.Generator().manual_seed(seed)
        hd = self.heads * self.dim
        self.a2 = (torch.randn((hd, self.rank), generator=g) * 1.5).to(dtype)
        self.bias = torch.randn(hd, generator=g) * 2.0 + 1.0
        if forget is not None:
            self.bias = torch.where(torch.arange(hd) % 3 == 0, torch.full((hd,), float(forget)), self.bias)
        self.norm = 1 + 0.4 * torch.randn(self.vdim, generator=g)
        self.dtype = dtype
        self.width = 2 * hd + 2 * self.heads * self.vdim + self.rank

    def inputs(self, T, seed):
        g = torch.Generator().manual_seed(seed)
        return (torch.randn((T, self.width), generator=g).to(self.dtype),)

    def plain(self, inputs, eps):
        x = inputs[0].double()
        hd, vv = self.heads * self.dim, self.heads * self.vdim
        z = x[:, 2 * hd + 2 * vv:] @ self.a2.double().T + self.bias.double()
        m = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}
        return plain.gla_of_projections(x[:, :hd], x[:, hd:2 * hd], x[:, 2 * hd:2 * hd + vv], x[:, 2 * hd + vv:2 * hd + 2 * vv], z, m,
                                        self.norm.double(), eps)

    def states(self, dev, slots, fill=float("nan")):
        return (torch.full((slots, self.heads, self.dim, self.vdim), fill, device=dev),)

    def run(self, k, dev, inputs, eps, states, q_lens, starts, slots):
        x = inputs[0]
        pad = -x.shape[1] % 8                                    # (a wider row, as the packed product makes it)
        x = torch.cat((x, torch.full((x.shape[0], pad), float("nan"), dtype=x.dtype)), dim=1)
        out = k.gated_linear(x.to(dev), self.heads, self.dim, self.vdim, self.a2.to(dev), self.bias.to(dev), self.tau, self.norm.to(dev),
                             eps, states[0], state_batch(dev, q_lens, starts, slots))
        k.check_faults()
        return out


class MatrixRule:
    """A matrix memory: shape (heads, dim, vdim, cap)."""
    def __init__(self, shape, seed, dtype, forget=None):
        self.heads, self.dim, self.vdim, self.cap = shape
        g = torch.Generator().manual_seed(seed)
        self.bias = torch.randn(2 * self.heads, generator=g)
        self.bias[self.heads:] += 2.0
        if forget is not None:
            self.bias[self.heads:] = float(forget)
        self.norm = 1 + 0.4 * torch.randn(self.heads * self.vdim, generator=g)
        self.dtype = dtype
        self.width = 2 * self.heads * (self.dim + self.vdim)

    def inputs(self, T, seed):
        g = torch.Generator().manual_seed(seed)
        return torch.randn((T, self.width), generator=g).to(self.dtype), torch.randn((T, 2 * self.heads), generator=g) * 2.0

    def plain(self, inputs, eps):
        x, gates = (t.double() for t in inputs)
        hd, vv = self.heads * self.dim, self.heads * self.vdim
        z = gates + self.bias.double()
        m = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.cap}
        return plain.matrix_memory_of_projections(x[:, :hd], x[:, hd:2 * hd], x[:, 2 * hd:2 * hd + vv], x[:, 2 * hd + vv:], z[:, :self.heads],
                                                  z[:, self.heads:], m, self.norm.double(), eps)

    def states(self, dev, slots, fill=float("nan")):
        full = lambda *shape: torch.full((slots, self.heads) + shape, fill, device=dev)
        return full(self.dim, self.vdim), full(self.dim), full()

    def run(self, k, dev, inputs, eps, states, q_lens, starts, slots):
        x, gates = inputs
        out = k.matrix_memory(x.to(dev), gates.to(dev).contiguous(), self.bias.to(dev), self.heads, self.dim, self.vdim, self.cap,
                              self.norm.to(dev), eps, *states, state_batch(dev, q_lens, starts, slots))
        k.check_faults()
        return out


def rule(kind, shape, seed, dtype, forget=None):
    return (LinearRule if kind == "linear" else MatrixRule)(shape, seed, dtype, forget)


def run_in_portions(r, k, dev, inputs, eps, states, portions, slot):
    outs, pos = [], 0
    for n in portions:
        outs.append(r.run(k, dev, tuple(t[pos:pos + n] for t in inputs), eps, states, [n], [pos], [slot]))
        pos += n
    return torch.cat(outs)
