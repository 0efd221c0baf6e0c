"""Nemidra: every mechanism alone, and the model through the step function and the engine, against
the plain implementation (tests/plain_nemidra.py).  Each test runs on the CPU stand-ins of the
device operations (tests/torch_kernels.py; this checks the stand-ins and the host logic) and, marked
gpu, on the HIP kernels."""
import json

import pytest
import torch

import helpers as H
import nemidra_cases as K
import plain_nemidra as plain
from nano_vllm_amd import LLM, SamplingParams
from nano_vllm_amd.config import ConfigError, NemidraConfig, architecture_of
from nano_vllm_amd.parts import BuildContext, PartSpec, make_part
from nano_vllm_amd.parts.base import NormedAddend, ScaledPair, StreamAddend
from torch_kernels import TorchKernels, new_caches

BACKENDS = ["cpu", pytest.param("hip", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
_hip = {}


def _kernels(backend, dtype=torch.float32):
    if backend == "cpu":
        return TorchKernels("cpu", dtype), "cpu"
    from nano_vllm_amd.kernels import HipKernels
    if dtype not in _hip:
        _hip[dtype] = HipKernels("cuda:0", dtype, quiet=True)
    return _hip[dtype], "cuda:0"


def _tol(dtype):
    return 3e-5 if dtype == torch.float32 else 2e-2


def _close(got, want, dtype, what="", tol=None):
    e = float((got.double().cpu() - want.double()).abs().max() / max(float(want.double().abs().max()), 1e-9))
    assert e < (tol or _tol(dtype)), f"{what}: differs by {e:.2e} of the largest"


# ------------------------------------------------------------------------------ configuration
def test_config_is_read_written_and_refused():
    for name, c in K.CONFIGS.items():
        d = c["cfg"].to_dict()
        arch = architecture_of(d)
        assert arch.name == "Nemidra"
        again = arch.parse_config(json.loads(json.dumps(d)))
        assert again == c["cfg"].__class__(**{**c["cfg"].__dict__, "dtype": again.dtype}), name
    d = K.CONFIGS["a"]["cfg"].to_dict()
    # what may be left out: the loop, the mask, the scales, the feed-forward, the shared expert, the router's scale, the rank
    e = json.loads(json.dumps(d))
    e.pop("loop"), e["layers"][1]["mixer"]["left"].pop("mask"), e["layers"][0].pop("mlp"), e["layers"][1]["mlp"].pop("shared")
    e["layers"][1]["mixer"].pop("left_scale"), e["layers"][1]["mlp"]["router"].pop("scale"), e["layers"][0]["mixer"].pop("decay_rank")
    got = NemidraConfig.from_dict(e)
    assert got.loop == (0, 4, 1) and got.layers[1].mixer.left.window is None and got.layers[0].mlp is None
    assert got.layers[1].mlp.shared_ff is None and got.layers[1].mixer.left_scale == 1.0 and got.layers[1].mlp.scale == 1.0
    assert got.layers[0].mixer.decay_rank is None
    spec = architecture_of(d).build_spec(K.CONFIGS["a"]["cfg"])
    assert [(r.layer, r.add_embedding) for r in spec.order] == [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    spec = architecture_of(d).build_spec(K.CONFIGS["c"]["cfg"])
    assert [(r.layer, r.add_embedding) for r in spec.order] == [(0, False), (0, True), (0, True), (1, False), (2, False), (3, False)]

    def broken(change):
        x = json.loads(json.dumps(d))
        change(x)
        with pytest.raises(ConfigError):
            NemidraConfig.from_dict(x)
    broken(lambda x: x["layers"][0].update(type="delta"))
    broken(lambda x: x["layers"][1]["mixer"]["left"].update(heads=3))           # 3 heads on 2 kv heads
    broken(lambda x: x["layers"][1]["mixer"].pop("right"))
    broken(lambda x: x["layers"][1]["mixer"]["right"].update(gate_cap=0.0))
    broken(lambda x: x["layers"][1]["mixer"]["right"].pop("gate_cap"))
    broken(lambda x: x["layers"][0]["mixer"].update(tau=-1.0))
    broken(lambda x: x["layers"][1]["mlp"]["router"].update(top=7))
    broken(lambda x: x["layers"][1]["mlp"].update(kind="mixture"))
    broken(lambda x: x["loop"].update(stop=5))
    broken(lambda x: x["loop"].update(start=3))
    broken(lambda x: x["loop"].update(times=0))
    broken(lambda x: x["embedding"]["bigram"].update(buckets=0))
    broken(lambda x: x["token_side"].update(dim=0))
    broken(lambda x: x.update(logit_softcap=0.0))
    broken(lambda x: x["norm"].update(eps=0.0))
    broken(lambda x: x.pop("max_positions"))
    broken(lambda x: x.pop("vocab"))


def test_the_checkpoint_is_read_by_its_own_names():
    from safetensors import safe_open
    with safe_open(K.model_folder("a") + "/model.safetensors", "pt", "cpu") as f:
        names = set(f.keys())
        shapes = {n: tuple(f.get_slice(n).get_shape()) for n in names}
    common = {"norm1", "norm1b", "side.gate", "side.proj", "side.norm"}
    ff = {"norm2", "norm2b"}
    gla = {"mix." + n for n in ("q", "k", "v", "g", "o", "norm", "a1", "a2", "a2.b")}
    pair = {"mix.left." + n + b for n in "qkvo" for b in ("", ".b")} | \
        {"mix.right." + n for n in ("q", "k", "v", "g", "o", "norm", "i", "i.b", "f", "f.b")}
    moe = lambda n: {"mlp.router"} | {f"mlp.e{e}.{m}" for e in range(n) for m in ("gate", "up", "down")}
    shared = {"mlp.shared." + n for n in ("gate", "up", "down", "sg")}
    want = {"embed", "bigram", "pos", "side.embed", "head", "final.norm"}
    want |= {"l0." + n for n in common | ff | gla | {"mlp.up", "mlp.down"}} | {"l1." + n for n in common | ff | pair | moe(6) | shared}
    want |= {"l2." + n for n in common | ff | gla | moe(5)} | {"l3." + n for n in common | pair}
    assert names == want, names ^ want
    assert shapes["bigram"] == (90, 48) and shapes["pos"] == (300, 48) and shapes["side.embed"] == (200, 40)
    assert shapes["l0.mix.a1"] == (5, 48) and shapes["l0.mix.a2"] == (42, 5) and shapes["l0.mix.a2.b"] == (42,)
    assert shapes["l1.mix.right.norm"] == (42,) and shapes["l0.mix.norm"] == (10,) and shapes["l1.mix.right.i"] == (3, 48)
    # the decay's first step rides in the packed projection, whose rows are whole vectors; the rank is the tensors'
    r = _runner("a", "cpu", "float32", 8)
    w = r.model.params["l0.mix.proj.weight"]
    rows = 2 * 3 * (14 + 10)
    assert w.shape[0] % 8 == 0 and torch.equal(w[rows:rows + 5], r.model.params["l0.mix.a1.weight"])
    assert float(w[rows + 5:].abs().sum()) == 0.0
    cfg = json.load(open(K.model_folder("a") + "/config.json"))
    for layer in cfg["layers"]:
        layer["mixer"].pop("decay_rank", None)
    assert NemidraConfig.from_dict(cfg).layers[0].mixer.decay_rank is None


def test_a_rank_that_no_configuration_names_is_the_tensors(tmp_path):
    import os
    import shutil
    folder = str(tmp_path / "m")
    shutil.copytree(K.model_folder("a"), folder)
    path = os.path.join(folder, "config.json")
    cfg = json.load(open(path))
    for layer in cfg["layers"]:
        layer["mixer"].pop("decay_rank", None)
    json.dump(cfg, open(path, "w"))
    toks = H.random_tokens(200, 20, 3)
    kernels, dev = _kernels("cpu")
    r = H.make_runner(folder, "float32", 8, 8, device=dev, kernels=kernels, max_requests=1)
    assert K.err(H.run_portions(r, "x", toks, [20]), K.plain_logits(K.model_folder("a"), toks)) < MODEL_TOL["float32"]


# ------------------------------------------------------------------------------ the embedding
def _embed_batch(dev, q_lens, starts, slots):
    return K.state_batch(dev, q_lens, starts, slots)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("buckets,mul_prev,mul_cur,vocab,width", [(89, 7, 3, 60, 48), (1, 5, 2, 30, 20), (1013, 40503, 0, 3000, 130),
                                                                  (997, 2000000011, 1999999973, 5000, 24)])
def test_three_embeddings_and_the_token_before(backend, dtype, buckets, mul_prev, mul_cur, vocab, width):
    """Whole, token by token, in portions, unequal requests in one batch, a slot that another request left: a first token
    has the table's last row, every other one the row of the token before it, wherever a portion was cut."""
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(buckets)
    table, bigram, pos = ((torch.randn((n, width), generator=g)).to(dtype) for n in (vocab, buckets + 1, 64))
    cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
    w = {"embed": table.double(), "bigram": bigram.double(), "pos": pos.double()}
    before = torch.full((4, 1), vocab - 1, dtype=torch.int32, device=dev)
    toks = {r: torch.randint(vocab // 2, vocab, (n,), generator=g).tolist() for r, n in (("a", 40), ("b", 3), ("c", 21))}
    slot = {"a": 2, "b": 0, "c": 0}
    steps = [[("b", 0, 1), ("a", 0, 17)], [("b", 1, 1), ("a", 17, 2)], [("b", 2, 1), ("a", 19, 1)], [("a", 20, 1)],
             [("c", 0, 9), ("a", 21, 18)], [("c", 9, 1), ("a", 39, 1)], [("c", 10, 11)]]       # c takes b's slot
    got = {r: [] for r in toks}
    for step in steps:
        step = sorted(step, key=lambda e: e[2] != 1)
        ids = [t for r, s, n in step for t in toks[r][s:s + n]]
        batch = _embed_batch(dev, [n for _, _, n in step], [s for _, s, _ in step], [slot[r] for r, _, _ in step])
        x = k.summed_embedding(table.to(dev), torch.tensor(ids, dtype=torch.int32, device=dev), bigram.to(dev), (buckets, mul_prev, mul_cur),
                               pos.to(dev), before, batch)
        assert x.dtype == torch.float32
        at = 0
        for r, s, n in step:
            got[r].append(x[at:at + n].cpu())
            at += n
    k.check_faults()
    for r in toks:
        _close(torch.cat(got[r]), plain.embed(cfg, w, toks[r]), torch.float32, r, tol=1e-6)
    assert int(before[1, 0]) == vocab - 1 and int(before[3, 0]) == vocab - 1          # other requests' slots
    # without the second and third table
    x = k.summed_embedding(table.to(dev), torch.tensor([3, 5], dtype=torch.int32, device=dev), None, None, None, None,
                           _embed_batch(dev, [2], [0], [0]))
    assert torch.equal(x.cpu(), table[[3, 5]].float())
    assert torch.equal(k.copy_rows(x), x)


# ------------------------------------------------------------------------------ norms into and of the stream
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 20), (5, 48), (3, 1030), (9, 2048), (70, 4096), (2, 9000)])
def test_addends_through_norms_with_offsets(backend, dtype, rows, width):
    """A sublayer's output, or a pair of them with a constant each, through a norm of its own (with an offset or without)
    into the float stream, with and without a float addend beside it; then the stream's norm, or none."""
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(width)
    draw = lambda *s: torch.randn(s, generator=g)
    a, b = draw(rows, width).to(dtype), (draw(rows, width) * 3).to(dtype)
    a[0] *= 0.001                                                    # (the eps inside the root counts)
    wa, w = (0.3 * draw(width)).to(dtype), (0.3 * draw(width)).to(dtype)
    r0, extra = draw(rows, width) * 2, draw(rows, width)
    for offset_a, offset, pair, more, norm in ((1.0, 1.0, False, False, True), (0.0, 1.0, False, True, True), (1.0, 1.0, True, False, True),
                                               (1.0, 0.0, True, True, True), (1.0, 0.0, True, True, False), (0.0, 0.0, False, False, False)):
        x = ScaledPair(a.to(dev), b.to(dev), 0.7, -1.3, k) if pair else a.to(dev)
        addends = (NormedAddend(x, wa.to(dev), 1e-3, 0.9, offset_a),) + ((StreamAddend(extra.to(dev)),) if more else ())
        res = r0.clone().to(dev)
        if norm:
            y, out = k.stream_rms_norm(addends, res, w.to(dev), 1e-4, offset)
        else:
            y, out = k.stream_add(addends, res)
        u = 0.7 * a.double() - 1.3 * b.double() if pair else a.double()
        want = r0.double() + 0.9 * plain.unit(u, 1e-3) * (offset_a + wa.double()) + (extra.double() if more else 0.0)
        assert out.data_ptr() == res.data_ptr() and y.dtype == dtype
        _close(out, want, torch.float32, "stream", tol=3e-6)
        _close(y, plain.unit(want, 1e-4) * (offset + w.double()) if norm else want, dtype, (offset_a, offset, pair, more, norm))
    if backend == "hip":
        _close(ScaledPair(a.to(dev), b.to(dev), 0.7, -1.3, k).tensor(), 0.7 * a.double() - 1.3 * b.double(), dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("tokens", [1, 5, 16])
def test_consumers_add_up_a_products_partial_sums(tokens):
    """A product of few rows whose k is split stays as partial sums: the stream's norm (alone and in a pair, with a bias),
    the token table's activation and the matrix memory's gates give from them what they give from the finished product."""
    from nano_vllm_amd.kernels.ops import SplitSum
    k, dev = _kernels("hip", torch.bfloat16)
    g = torch.Generator().manual_seed(tokens)
    x = torch.randn((tokens, 1024), generator=g).to(torch.bfloat16).to(dev)
    mat = lambda n: (torch.randn((n, 1024), generator=g) / 32.0).to(torch.bfloat16).to(dev)
    vec = lambda n: (0.2 * torch.randn(n, generator=g)).to(torch.bfloat16).to(dev)
    a, b = k.linear(x, mat(256), vec(256), deferred=True), k.linear(x, mat(256), deferred=True)
    assert isinstance(a, SplitSum) and isinstance(b, SplitSum)
    wa, w, r0 = vec(256), vec(256), torch.randn((tokens, 256), generator=g).to(dev)
    for p, q in (((a, None), (a.tensor(), None)), ((a, b), (a.tensor(), b.tensor())), ((a, b), (a.tensor(), b)), ((a, b), (a, b.tensor()))):
        outs = []
        for left, right in (p, q):
            add = NormedAddend(left if right is None else ScaledPair(left, right, 0.5, 2.0, k), wa, 1e-5, 1.0, 1.0)
            outs.append(k.stream_rms_norm((add,), r0.clone(), w, 1e-5, 1.0))
        assert torch.equal(outs[0][0], outs[1][0]) and torch.equal(outs[0][1], outs[1][1])
    assert torch.equal(ScaledPair(a, b, 0.5, 2.0, k).tensor(), ScaledPair(a.tensor(), b.tensor(), 0.5, 2.0, k).tensor())
    z = k.linear(x, mat(32), deferred=True)
    assert isinstance(z, SplitSum)
    table, ids = torch.randn((50, 96), generator=g).to(torch.bfloat16).to(dev), torch.randint(0, 50, (tokens,), generator=g).to(torch.int32).to(dev)
    assert torch.equal(k.act_mul_rows(z, table, ids, 32), k.act_mul_rows(z.tensor(), table, ids, 32))
    gates = k.linear(x, mat(8), out_float32=True, deferred=True)
    assert isinstance(gates, SplitSum) and gates.dtype == torch.float32
    rule = K.rule("matrix", (4, 16, 8, 5.0), 3, torch.bfloat16)
    proj = rule.inputs(tokens, 4)[0]
    found = []
    for gt in (gates, gates.tensor()):
        states = rule.states(dev, tokens, 0.5)
        out = k.matrix_memory(proj.to(dev), gt, rule.bias.to(dev), 4, 16, 8, 5.0, rule.norm.to(dev), 1e-5, *states,
                              K.state_batch(dev, [1] * tokens, [1] * tokens, list(range(tokens))))
        found.append((out.float(), *states))
    for p, q in zip(*found):
        assert torch.allclose(p, q, rtol=1e-2, atol=1e-5)


# ------------------------------------------------------------------------------ the tokens' table, activations, the cap
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
def test_the_layers_part_of_the_tokens_row(backend, dtype):
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(5)
    table = torch.randn((40, 36), generator=g).to(dtype)
    x = (torch.randn((7, 12), generator=g) * 2).to(dtype)
    ids = [0, 39, 5, 5, 17, 1, 38]
    for part in range(3):
        got = k.act_mul_rows(x.to(dev), table.to(dev), torch.tensor(ids, dtype=torch.int32, device=dev), 12 * part, "gelu_tanh")
        _close(got, plain.gelu_tanh(x.double()) * table[ids, 12 * part:12 * part + 12].double(), dtype, part)
    # the whole sublayer, through its part
    build = BuildContext(k, torch.device(dev), dtype, 24, 64)
    build.tables["t"] = make_part("table", PartSpec("token_table", {"rows": 40, "width": 36}), build)
    build.tables["t"].weights["weight"] = table.to(dev)
    part = make_part("token_side", PartSpec("token_side", {"hidden_size": 24, "dim": 12, "offset": 24, "table": "t", "activation": "gelu_tanh",
                                                           "norm": PartSpec("rms_norm", {"dim": 24, "eps": 1e-5})}), build)
    w = {"gate.weight": torch.randn((12, 24), generator=g) * 0.3, "proj.weight": torch.randn((24, 12), generator=g) * 0.3}
    part.weights.update({n: t.to(dtype).to(dev) for n, t in w.items()})
    r = (torch.randn((7, 24), generator=g)).to(dtype)
    got = part.forward(r.to(dev), torch.tensor(ids, dtype=torch.int32, device=dev))
    got = got.tensor() if hasattr(got, "tensor") else got
    want = (plain.gelu_tanh(r.double() @ w["gate.weight"].to(dtype).double().T) * table[ids, 24:36].double()) @ w["proj.weight"].to(dtype).double().T
    _close(got, want, dtype, "sublayer")


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,width,inner", [(1, 48, 36), (3, 520, 72), (40, 128, 192), (300, 64, 40), (8, 512, 8192)])
def test_the_exact_gelu_after_a_product(backend, dtype, tokens, width, inner):
    """The exact form, which differs from the tanh form by up to 5e-4: float32 tells them apart."""
    if backend == "cpu" and inner > 1000:
        pytest.skip("a size of the wide product's kernel")
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(tokens)
    x = torch.randn((tokens, width), generator=g).to(dtype)
    w = (torch.randn((inner, width), generator=g) * 2 / width ** 0.5).to(dtype)
    got = k.linear_act(x.to(dev), w.to(dev), "gelu") if backend == "hip" else k.act(k.linear(x, w), "gelu")
    _close(got, plain.gelu_erf(x.double() @ w.double().T), dtype)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [97, 580, 4096])
def test_capped_logits(backend, width):
    k, dev = _kernels(backend)
    x = torch.linspace(-200.0, 200.0, 5 * width).view(5, width)
    got = k.softcap_(x.clone().to(dev), 25.0)
    _close(got, 25.0 * torch.tanh(x.double() / 25.0), torch.float32, tol=1e-6)


# ------------------------------------------------------------------------------ experts
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top", [(6, 2), (1, 1), (4, 4), (70, 5), (300, 8)])
def test_softmax_scores_choose_and_weigh(backend, experts, top):
    """The weights are the scores over all experts times the scale, not over the chosen ones' sum; equal scores go to the
    lower number."""
    k, dev = _kernels(backend)
    g = torch.Generator().manual_seed(experts)
    z = torch.randn((50, experts), generator=g) * 3
    if experts > 1:
        z[7] = 1.0
        z[8] += 80.0                                                  # (a softmax without its maximum taken off would overflow)
    ids, weights = k.moe_route(z.to(dev), top, 1, 1, 1.7, routing="softmax_scores")
    for t in range(50):
        if t == 7 and backend == "cpu":
            continue
        want = plain.choose(z[t].double(), {"top": top, "scale": 1.7})
        assert [int(e) for e in ids[t].cpu()] == [e for e, _ in want], t
        for got, (_, w) in zip(weights[t].cpu(), want):
            assert abs(float(got) - w) < 2e-6 * max(w, 1e-3), t


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,ff,shared,hidden,tokens", [(6, 2, 20, 28, 48, 33), (1, 1, 6, 1, 20, 4), (4, 4, 5, None, 20, 9), (8, 2, 64, 64, 128, 200)])
def test_the_routed_feed_forward(backend, dtype, experts, top, ff, shared, hidden, tokens):
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(experts + hidden)
    names = {"gate_name": "gate", "up_name": "up", "down_name": "down"}
    build = BuildContext(k, torch.device(dev), dtype, hidden, 64)
    sp = None if shared is None else PartSpec("swiglu", {"hidden_size": hidden, "intermediate_size": shared, **names})
    part = make_part("feed_forward", PartSpec("moe", {
        "hidden_size": hidden, "num_experts": experts, "top": top, "intermediate_size": ff, "scale": 1.4, "routing": "softmax_scores",
        "gated": True, "activation": "silu", "shared": sp, "shared_gate": sp is not None, "router_name": "router", "expert_name": "e{}",
        "shared_name": "shared", "shared_gate_name": "sg", **names}), build)
    draw = lambda *s: (torch.randn(s, generator=g) * 0.4).to(dtype)
    w = {"router": draw(experts, hidden)}
    for e in range(experts):
        w.update({f"e{e}.gate": draw(ff, hidden), f"e{e}.up": draw(ff, hidden), f"e{e}.down": draw(hidden, ff)})
    if shared is not None:
        w.update({"shared.gate": draw(shared, hidden), "shared.up": draw(shared, hidden), "shared.down": draw(hidden, shared), "shared.sg": draw(1, hidden)})
        part.shared.weights["gate_up_proj.weight"] = torch.cat((w["shared.gate"], w["shared.up"])).to(dev)
        part.shared.weights["down.weight"] = w["shared.down"].to(dev)
    part.weights["router.weight"] = torch.cat([w["router"]] + ([w["shared.sg"]] if shared is not None else [])).to(dev)
    part.weights["up.weight"] = torch.cat([w[f"e{e}.{m}"] for e in range(experts) for m in ("gate", "up")]).to(dev)
    part.weights["down.weight"] = torch.cat([w[f"e{e}.down"] for e in range(experts)]).to(dev)
    x = torch.randn((tokens, hidden), generator=g).to(dtype)
    got = part.forward(x.to(dev))
    mlp = {"router": {"top": top, "scale": 1.4}, "shared": None if shared is None else {"ff": shared}}
    want = plain.experts(x.double(), mlp, {n: t.double() for n, t in w.items()}, "")
    _close(got, want, dtype, tol=3e-2 if dtype == torch.bfloat16 else None)


# ------------------------------------------------------------------------------ the window attention
def _window_run(k, dev, dtype, hq, hkv, D, DV, page, lens, q_lens, window, scale, q, kk, vv, seed=7, free_passed=True):
    batch, _, all_slots, pages = K.paged_batch(dev, page, lens, q_lens, seed, window, free_passed)
    kc, vc = new_caches(pages, hkv, D, page, dtype, dev, v_head_dim=DV)
    kc.fill_(float("nan")), vc.fill_(float("nan"))
    for s in range(len(lens)):
        K.fill_cache(kc, vc, all_slots[s], kk[s], vv[s])
    qs = torch.cat([q[s][n - c:].reshape(c, hq * D) for s, (n, c) in enumerate(zip(lens, q_lens))])
    out = k.paged_attention(qs.to(dev), hq, hkv, D, kc, vc, batch, 0, scale, window, v_head_dim=DV)
    k.check_faults()
    return out


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hq,hkv,D,DV,page,window,lens,q_lens", [
    (4, 2, 12, 16, 8, 10, [30, 9, 41], [1, 1, 41]),
    (3, 1, 6, 10, 4, 1, [13, 6], [1, 6]),
    (6, 3, 24, 24, 16, 33, [50, 33], [17, 33]),
    (6, 2, 40, 40, 64, 70, [200, 3, 130], [1, 2, 130]),            # a head size that the matrix cores' kernels leave to the general one
    (8, 2, 64, 64, 32, 48, [130, 70, 100], [1, 2, 64]),
])
def test_window_attention_over_pages(backend, dtype, hq, hkv, D, DV, page, window, lens, q_lens):
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(D)
    draw = lambda n, h, d: torch.randn((n, h, d), generator=g).to(dtype)
    q, kk, vv = ([draw(n, h, d) for n in lens] for h, d in ((hq, D), (hkv, D), (hkv, DV)))
    got = _window_run(k, dev, dtype, hq, hkv, D, DV, page, lens, q_lens, window, 0.3, q, kk, vv)
    want = torch.cat([plain.window_attend(a.double(), b.double(), c.double(), 0.3, window, rows=range(n - m, n))[n - m:].reshape(m, -1)
                      for a, b, c, n, m in zip(q, kk, vv, lens, q_lens)])
    _close(got, want, dtype)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,DV,page,window", [(12, 8, 8, 23), (40, 40, 32, 64), (40, 56, 64, 65), (64, 64, 32, 23)])
def test_a_key_just_inside_and_just_outside_the_window(backend, dtype, D, DV, page, window):
    """One key takes nearly all the weight of the queries whose window holds it: the last query of a portion, of a whole
    prompt, and a single token follow it at the window's oldest place, and take nothing of it one place further."""
    k, dev = _kernels(backend, dtype)
    for n, portion in ((230, 1), (230, 40), (130, 130)):
        for back in (0, window - 1, window):
            j = n - 1 - back
            q, kk, vv = torch.zeros((n, 2, D)), torch.zeros((n, 1, D)), torch.zeros((n, 1, DV))
            q[:, :, 1] = 6.0
            kk[j, 0, 1] = 6.0
            vv[:, 0, 0], vv[j, 0, 0], vv[j, 0, 1] = 1.0, 0.0, 1.0
            got = _window_run(k, dev, dtype, 2, 1, D, DV, page, [n], [portion], window, 0.5, [q.to(dtype)], [kk.to(dtype)], [vv.to(dtype)])
            last = got[-1].float().cpu().view(2, DV)
            seen = 1.0 if back < window else 0.0
            assert float((last[:, 1] - seen).abs().max()) < 1e-2 and float((last[:, 0] - (1.0 - seen)).abs().max()) < 1e-2, (n, portion, back)


# ------------------------------------------------------------------------------ the two state layers
RULES = [("linear", (3, 14, 10, 5, 4.0)), ("linear", (1, 1, 1, 1, 1.0)), ("linear", (2, 64, 64, 16, 16.0)), ("linear", (1, 130, 20, 3, 8.0)),
         ("linear", (2, 40, 72, 24, 0.5)), ("linear", (1, 128, 256, 8, 16.0)), ("linear", (1, 20, 260, 4, 16.0)), ("linear", (1, 260, 12, 4, 16.0)),
         ("matrix", (3, 10, 14, 5.0)), ("matrix", (1, 1, 1, 1.0)), ("matrix", (2, 64, 64, 15.0)), ("matrix", (1, 130, 20, 8.0)),
         ("matrix", (2, 40, 72, 12.0)), ("matrix", (1, 200, 250, 12.0)), ("matrix", (1, 20, 260, 8.0)), ("matrix", (1, 260, 12, 8.0))]


def _state_tol(dtype):
    return 4e-2 if dtype == torch.bfloat16 else 1e-4


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,shape", RULES)
def test_a_state_layer_in_portions_of_every_size_and_token_by_token(backend, dtype, kind, shape):
    """One request: whole, token by token, and in portions down to two tokens, on a slot that held NaN (a request's
    start reads nothing of what its slot held)."""
    if backend == "cpu" and dtype == torch.bfloat16 and shape[1] >= 40:
        pytest.skip("the same path as float32 on the stand-ins")
    k, dev = _kernels(backend, dtype)
    T, eps = 45, 1e-5
    r = K.rule(kind, shape, 11, dtype)
    inputs = r.inputs(T, 12)
    want = r.plain(inputs, eps)
    cuttings = ([T], [1] * T, [2, 2, 1, 3, 1, 1, 2, 17, 5, 2, 9], [1, 44], [44, 1], [13, 2, 30], [16, 16, 13], [15, 17, 13])
    for portions in cuttings[:3] if backend == "cpu" and shape[1] >= 40 else cuttings:
        states = r.states(dev, 3)
        _close(K.run_in_portions(r, k, dev, inputs, eps, states, portions, 1), want, dtype, portions[:4], _state_tol(dtype))
        for s in states:
            assert torch.isnan(s[0]).all() and torch.isnan(s[2]).all(), "another request's slot was written"


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("kind,shape", [RULES[0], RULES[8]])
def test_a_state_layer_of_unequal_requests_in_one_batch(backend, kind, shape):
    """Steps of requests of unequal lengths (single tokens first, as the batch orders them), on slots in another order
    than the requests; one request ends and another takes its slot."""
    k, dev = _kernels(backend)
    eps = 1e-6
    r = K.rule(kind, shape, 21, torch.float32)
    lens = {"a": 30, "b": 3, "c": 55, "d": 17, "e": 26}
    inputs = {q: r.inputs(n, 30 + i) for i, (q, n) in enumerate(lens.items())}
    want = {q: r.plain(inputs[q], eps) for q in lens}
    states = r.states(dev, 4)
    slot = {"a": 2, "b": 0, "c": 3, "d": 1, "e": 0}
    steps = [[("b", 0, 1), ("a", 0, 30), ("c", 0, 20), ("d", 0, 2)],
             [("b", 1, 1), ("d", 2, 1), ("c", 20, 33)],
             [("b", 2, 1), ("c", 53, 1), ("d", 3, 14)],
             [("c", 54, 1), ("e", 0, 26)]]                              # e takes b's slot, which holds b's last state
    got = {q: [] for q in lens}
    for step in steps:
        part = tuple(torch.cat([inputs[q][i][s:s + n] for q, s, n in step]) for i in range(len(inputs["a"])))
        out = r.run(k, dev, part, eps, states, [n for _, _, n in step], [s for _, s, _ in step], [slot[q] for q, _, _ in step])
        row = 0
        for q, s, n in step:
            got[q].append(out[row:row + n])
            row += n
    for q in lens:
        _close(torch.cat(got[q]), want[q], torch.float32, q, 1e-4)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,shape", [RULES[0], RULES[2], RULES[4], RULES[8], RULES[10], RULES[12]])
def test_long_portions_beside_single_tokens(backend, dtype, kind, shape):
    """Portions of one unit, exactly one, one token more and several beside single tokens, from a start and from a state:
    outputs are the plain implementation's, and the states are those of the walk token by token."""
    k, dev = _kernels(backend, dtype)
    if backend == "cpu" and (dtype == torch.bfloat16 or shape[1] >= 40):
        pytest.skip("the stand-ins run one way only")
    eps = 1e-5
    r = K.rule(kind, shape, 41, dtype)
    lens = {"a": 9, "b": 130, "c": 67, "d": 200, "e": 68, "f": 33, "g": 32}
    inputs = {q: r.inputs(n, 50 + i) for i, (q, n) in enumerate(lens.items())}
    want = {q: r.plain(inputs[q], eps) for q in lens}
    slot = {"a": 2, "b": 0, "c": 4, "d": 1, "e": 3, "f": 6, "g": 7}
    steps = [[("a", 0, 8), ("b", 0, 64), ("c", 0, 65), ("d", 0, 3), ("f", 0, 33), ("g", 0, 32)],
             [("a", 8, 1), ("b", 64, 1), ("d", 3, 131), ("c", 65, 2), ("e", 0, 67)],
             [("e", 67, 1), ("b", 65, 65), ("d", 134, 66)]]
    found = {}
    for blocks in (True, 64, False) if backend == "hip" else (True,):            # (64: units of that many tokens)
        if backend == "hip":
            k.memory_blocks, k.memory_unit_tokens = bool(blocks), 64 if blocks == 64 else 0
        try:
            states, got = r.states(dev, 8), {q: [] for q in lens}
            for step in steps:
                part = tuple(torch.cat([inputs[q][i][s:s + n] for q, s, n in step]) for i in range(len(inputs["a"])))
                out = r.run(k, dev, part, eps, states, [n for _, _, n in step], [s for _, s, _ in step], [slot[q] for q, _, _ in step])
                row = 0
                for q, s, n in step:
                    got[q].append(out[row:row + n])
                    row += n
            for q in lens:
                _close(torch.cat(got[q]), want[q], dtype, (q, blocks), _state_tol(dtype))
            assert all(torch.isnan(s[5]).all() for s in states)
            found[blocks] = states
        finally:
            if backend == "hip":
                k.memory_blocks, k.memory_unit_tokens = True, 0
    if backend == "hip":
        # the states agree far below what bfloat16's outputs show (linear: the portions' decay logits come from another product)
        held = [s for s in range(8) if s != 5]
        for other in (True, 64):
            for a, b in zip(found[other], found[False]):
                _close(a[held], b[held].cpu(), torch.float32, "states", 1e-4)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("kind,shape,forget", [("linear", (2, 20, 24, 4, 1.0), -30.0), ("linear", (1, 64, 64, 4, 0.25), -3.0), ("linear", (2, 20, 24, 4, 1.0), 60.0),
                                               ("matrix", (2, 20, 24, 40.0), -60.0), ("matrix", (2, 20, 24, 30.0), 90.0), ("matrix", (2, 20, 24, 1.0), -4.0)])
def test_channels_that_forget_at_once_and_channels_that_keep_all(backend, kind, shape, forget):
    """Decays of exp(-30) and far less a token beside slow ones (products of quotients of such decays leave the floats'
    range), and decays of one to the last bit; in portions over several units."""
    k, dev = _kernels(backend)
    T, eps = 150, 1e-6
    r = K.rule(kind, shape, 8, torch.float32, forget=forget)
    inputs = r.inputs(T, 9)
    want = r.plain(inputs, eps)
    for portions in ([T], [70, 1, 79], [2] * 5 + [140]):
        _close(K.run_in_portions(r, k, dev, inputs, eps, r.states(dev, 1), portions, 0), want, torch.float32, portions[:3], 2e-4)


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_matrix_memorys_maximum_starts_at_zero(backend):
    """Input gates far below zero and forget gates that keep: the running maximum stays where it started, the write factor
    is the gate itself and the divisor is the floor exp(-m), not |n.q|."""
    k, dev = _kernels(backend)
    r = K.rule("matrix", (2, 12, 8, 20.0), 3, torch.float32, forget=40.0)
    inputs = r.inputs(40, 5)
    inputs[1][:, :2] = -8.0
    inputs[1][20:22, :2] = 6.0                                        # then two tokens that raise it
    want = r.plain(inputs, 1e-2)                                      # (an eps that sees how large o is)
    for portions in ([40], [1] * 40, [19, 2, 19]):
        states = r.states(dev, 1)
        _close(K.run_in_portions(r, k, dev, inputs, 1e-2, states, portions, 0), want, torch.float32, portions[:3], 1e-4)
    wrong = inputs[1].clone()
    wrong[:, :2] += 1.0                                               # the oracle with other gates differs clearly
    assert float((r.plain((inputs[0], wrong), 1e-2) - want).abs().max()) > 1e-2 * float(want.abs().max())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("kind,shape", [("linear", (2, 16, 8, 4, 16.0)), ("linear", (1, 64, 64, 4, 16.0)), ("matrix", (2, 16, 8, 15.0)), ("matrix", (1, 64, 64, 15.0))])
def test_a_far_write_is_read_out(backend, kind, shape):
    """A value written at token 0 for a key that no later key touches is read out 400 tokens later, whole and in portions.
    The state is float32 and keeps it."""
    k, dev = _kernels(backend)
    T, eps = 400, 1e-6
    r = K.rule(kind, shape, 5, torch.float32)
    heads, dim, vdim = r.heads, r.dim, r.vdim
    inputs = r.inputs(T, 9)
    x = inputs[0]
    x[:, :2 * heads * dim] = 0
    for h in range(heads):
        x[:, h * dim + 5] = 1.0                              # every token asks for axis 5 ...
        x[-1, h * dim + 5], x[-1, h * dim + 3] = 0.0, 1.0    # ... the last one for axis 3
        x[:, (heads + h) * dim + 5] = 1.0                    # and writes there ...
        x[0, (heads + h) * dim + 5], x[0, (heads + h) * dim + 3] = 0.0, 1.0
    if kind == "linear":
        x[:, -r.rank:] = 0
        r.bias[:] = 9.0                                      # (a decay of exp(-1.2e-4 / 16) a token)
    else:
        inputs[1][:] = 0
        r.bias[:heads] = 0.0
        r.bias[heads:] = 12.0
    want = r.plain(inputs, eps)
    v0 = x[0, 2 * heads * dim:2 * heads * dim + vdim].double()
    gate = x[-1, 2 * heads * dim + heads * vdim:2 * heads * dim + heads * vdim + vdim].double()
    ahead = plain.unit(v0, eps) * r.norm[:vdim].double() * (plain.silu(gate) if kind == "linear" else torch.sigmoid(gate))
    assert float((want[-1, :vdim] - ahead).abs().max()) < 1e-2 * float(ahead.abs().max())
    for portions in ([T], [T - 1, 1], [150, 249, 1]):
        _close(K.run_in_portions(r, k, dev, inputs, eps, r.states(dev, 1), portions, 0)[-1], want[-1], torch.float32, portions, 1e-4)


def test_portions_are_cut_into_units():
    from nano_vllm_amd.kernels.ops import memory_units
    units, chains = memory_units([1, 1, 130, 2, 64], 2, 4, 256)
    assert units == [2, 2, 32, 1, 2, 34, 32, 1, 2, 66, 32, 1, 2, 98, 32, 1, 2, 130, 2, 2, 3, 132, 2, 0, 4, 134, 32, 1, 4, 166, 32, 2]
    assert chains == [0, 5, 2, 0, 6, 2, 4, 0]
    units, chains = memory_units([130, 2], 0, 4, 256, tokens=64)
    assert units == [0, 0, 64, 1, 0, 64, 64, 1, 0, 128, 2, 2, 1, 130, 2, 0] and chains == [0, 3, 0, 0]
    for n, heads in ((20000, 16), (100000, 32), (300, 2)):
        units, chains = memory_units([n], 0, heads, 256)
        sizes = units[2::4]
        assert sum(sizes) == n and all(s % 16 == 0 and s == sizes[0] for s in sizes[:-1]) and 0 < sizes[-1] <= sizes[0]
        assert units[1::4] == [i * sizes[0] for i in range(len(sizes))] and units[3::4] == [1] * (len(sizes) - 1) + [2]
        assert sizes[0] == 32 or len(sizes) * heads >= 256


# ------------------------------------------------------------------------------ the model through the step function
def _runner(name, backend, dtype, pages, max_requests=4):
    kernels, dev = _kernels(backend, torch.float32 if dtype == "float32" else torch.bfloat16)
    return H.make_runner(K.model_folder(name, dtype), dtype, K.CONFIGS[name]["page"], pages, device=dev,
                         kernels=kernels, max_requests=max_requests)


MODEL_TOL = {"float32": 2e-4, "bfloat16": 6e-2}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["a", "b", "c", "d"])
def test_every_cutting_gives_the_plain_logits(backend, name):
    c = K.CONFIGS[name]
    n = 70 if backend == "cpu" else 110
    toks = H.random_tokens(c["cfg"].vocab, n, 1)
    want = K.plain_logits(K.model_folder(name), toks)
    r = _runner(name, backend, "float32", 60)
    start, stop, times = c["cfg"].loop
    runs = len(c["cfg"].layers) + (times - 1) * (stop - start)
    assert len(r.layer_caches) == runs + 1                     # every pass has a cache of its own; the embedding keeps a token
    for portions in (H.whole(n), H.last_one_by_one(n, 45), H.changing_portions(n, 2), [1] * 3 + [2] * 10 + [n - 23]):
        got = H.run_portions(r, "x", toks, portions)
        assert K.err(got, want) < MODEL_TOL["float32"], portions
    assert all(pool.num_free == 60 for pool in r.cache.pools)


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["a", "b", "d"])
def test_bfloat16_follows_the_plain_logits_under_every_cutting(name):
    c = K.CONFIGS[name]
    n = 130
    toks = H.random_tokens(c["cfg"].vocab, n, 3)
    want = K.plain_logits(K.model_folder(name, "bfloat16"), toks)
    r = _runner(name, "hip", "bfloat16", 60)
    for portions in (H.whole(n), H.last_one_by_one(n, 40), H.changing_portions(n, 4)):
        e = K.errors(H.run_portions(r, "x", toks, portions), want)
        # (a token whose experts lie close may take another one)
        assert float(e.median()) < 0.06 and float(e.quantile(0.9)) < 0.2, (portions, float(e.median()), float(e.quantile(0.9)), float(e.max()))


@pytest.mark.gpu
def test_a_larger_model_over_long_prompts():
    """Six hundred tokens through a model with a window over several pages and states of several tiles: whole, in
    changing portions, and its last tokens one by one."""
    name = "e"
    c = K.CONFIGS[name]
    n = 600
    toks = H.random_tokens(c["cfg"].vocab, n, 17)
    want = K.plain_logits(K.model_folder(name), toks)
    r = _runner(name, "hip", "float32", 12)
    for portions in (H.whole(n), H.changing_portions(n, 5), H.last_one_by_one(n, 180)):
        assert K.err(H.run_portions(r, "x", toks, portions), want) < MODEL_TOL["float32"], portions[:4]
    assert all(pool.num_free == 12 for pool in r.cache.pools)
    want16 = K.plain_logits(K.model_folder(name, "bfloat16"), toks)
    r = _runner(name, "hip", "bfloat16", 12)
    for portions in (H.whole(n), H.changing_portions(n, 5), H.last_one_by_one(n, 60)):
        e = K.errors(H.run_portions(r, "x", toks, portions), want16)
        assert float(e.median()) < 0.06 and float(e.quantile(0.9)) < 0.2, (portions[:4], float(e.median()), float(e.quantile(0.9)))


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_first_tokens_of_a_sequence(backend):
    for name in ("a", "c"):
        c = K.CONFIGS[name]
        r = _runner(name, backend, "float32", 8)
        for n in (1, 2, 3, 5):
            toks = H.random_tokens(c["cfg"].vocab, n, 40 + n)
            want = K.plain_logits(K.model_folder(name), toks)
            for portions in ([n], [1] * n):
                assert K.err(H.run_portions(r, "x", toks, portions), want) < MODEL_TOL["float32"], (name, n, portions)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["a", "c"])
def test_long_decoding(backend, name):
    # 171 tokens one by one: every window passes over decoded tokens, the states run on from the first token
    c = K.CONFIGS[name]
    n = 171
    toks = H.random_tokens(c["cfg"].vocab, n, 5)
    want = K.plain_logits(K.model_folder(name), toks)
    r = _runner(name, backend, "float32", 48)
    assert K.err(H.run_portions(r, "x", toks, [1] * n), want) < MODEL_TOL["float32"]
    if name == "a":
        # a window's group holds the pages of its window only
        r.cache.admit("y")
        for pos in range(n):
            r.cache.reserve("y", pos + 1)
        by_window = {g.window: sum(1 for p in t if p >= 0) for g, t in zip(r.cache.groups, r.cache.requests["y"].tables)}
        assert by_window[10] <= 3 and by_window[21] <= 4, by_window
        r.cache.release("y")


def test_positions_beyond_the_table_are_refused():
    r = _runner("c", "cpu", "float32", 80)
    r.cache.admit("x")
    r.cache.reserve("x", 257)
    from nano_vllm_amd.engine.batch import StepEntry
    with pytest.raises(ValueError):
        r.step([StepEntry("x", [1], 256, [0])])
    r.cache.release("x")


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["a", "d"])
def test_mixed_batches_on_pages_and_slots_that_are_used_again(backend, name):
    c = K.CONFIGS[name]
    lens = {"r0": 60, "r1": 41, "r2": 77, "r3": 1, "r4": 35, "r5": 52, "r6": 66, "r7": 2}
    reqs = {r: H.random_tokens(c["cfg"].vocab, n, i) for i, (r, n) in enumerate(lens.items())}
    pages = 192 // c["page"]                   # 192 tokens of cache for 334 tokens of eight requests, three slots
    r = _runner(name, backend, "float32", pages, max_requests=3)
    got = H.run_mixed(r, reqs, seed=3, max_live=3)
    for rid, toks in reqs.items():
        assert K.err(got[rid], K.plain_logits(K.model_folder(name), toks)) < MODEL_TOL["float32"], rid
    assert all(pool.num_free == pages for pool in r.cache.pools)
    # each request alone gives what it gave in the batches
    alone = _runner(name, backend, "float32", pages, max_requests=1)
    for rid in ("r1", "r3", "r6"):
        one = H.run_portions(alone, rid, reqs[rid], [len(reqs[rid])])
        assert K.err(got[rid], one) < 4e-5, rid


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["a", "c"])
def test_the_residual_stream_after_every_layer(backend, name):
    """Layer run by layer run (a looped layer counts each time): the float32 stream after it is the plain implementation's.
    The stream takes a layer's last addend inside the norm that follows, so it is read where that norm leaves it; where a
    pass begins there, that norm has added the embedding too."""
    c = K.CONFIGS[name]
    toks = H.random_tokens(c["cfg"].vocab, 37, 9)
    cfg, w = K.plain_model(K.model_folder(name))
    _, streams = plain.forward(cfg, w, toks, return_layers=True)
    e0 = plain.embed(cfg, w, toks)
    r = _runner(name, backend, "float32", 12)
    seen = []
    inner = r.kernels.stream_rms_norm

    def spy(addends, residual, *a, **kw):
        y, res = inner(addends, residual, *a, **kw)
        seen.append(res.detach().float().cpu().clone())
        return y, res
    r.kernels.stream_rms_norm = spy
    try:
        H.run_portions(r, "x", toks, [len(toks)])
    finally:
        del r.kernels.stream_rms_norm
    order = plain.run_order(cfg)
    at, ends = 0, []
    for i, _ in order:
        at += 2 if cfg["layers"][i].get("mlp") else 1
        ends.append(at)                                   # the norm that first sees the stream after this run
    assert len(seen) == at + 1
    _close(seen[0], e0, torch.float32, "embedding")
    for n, want in enumerate(streams):
        if n + 1 < len(order) and order[n + 1][1]:
            want = want + e0
        assert float((seen[ends[n]].double() - want).abs().max() / want.abs().max()) < 3e-5, n


# ------------------------------------------------------------------------------ the engine
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("schedule", ["prefill_first", "mixed"])
def test_greedy_generation_through_the_engine(backend, schedule):
    name = "d"
    c = K.CONFIGS[name]
    kernels, dev = _kernels(backend)
    folder = K.model_folder(name)
    prompts = [H.random_tokens(c["cfg"].vocab, n, 60 + n) for n in (3, 30, 1, 47, 18)]
    # few pages, three requests at a time and portions of at most 16 tokens: prompts are cut, requests wait
    llm = LLM(folder, kernels=kernels, device=dev, dtype="float32", kvcache_block_size=c["page"], num_kvcache_blocks=10,
              max_num_batched_tokens=16, max_num_seqs=3, schedule=schedule, max_model_len=128)
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True), use_tqdm=False)
    cfg, w = K.plain_model(folder)
    for p, o in zip(prompts, outs):
        # (one pass of the plain implementation over prompt and answer: every answered token is its best one)
        best = K.plain_logits(folder, p + o["token_ids"][:-1])[len(p) - 1:].argmax(-1).tolist()
        assert o["token_ids"] == best, len(p)
    assert outs[2]["token_ids"][:3] == plain.greedy_generate(cfg, w, prompts[2], 3)
    assert all(pool.num_free == 10 for pool in llm.runner.cache.pools)


@pytest.mark.gpu
def test_generation_in_bfloat16_with_captured_steps_and_bursts():
    name = "b"
    c = K.CONFIGS[name]
    folder = K.model_folder(name, "bfloat16")
    prompts = [H.random_tokens(c["cfg"].vocab, n, 80 + n) for n in (5, 40, 90, 17)]
    sp = SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True)
    common = dict(dtype="bfloat16", kvcache_block_size=c["page"], num_kvcache_blocks=24, max_num_seqs=4, max_model_len=256)
    eager = LLM(folder, enforce_eager=True, **common).generate(prompts, sp, use_tqdm=False)
    graphs = LLM(folder, decode_burst=8, **common)
    assert graphs.runner._graph_max_batch, "nothing in the model's single-token step asks the host: its steps are captured"
    fast = graphs.generate(prompts, sp, use_tqdm=False)
    for a, b in zip(eager, fast):
        assert a["token_ids"] == b["token_ids"]


@pytest.mark.gpu
def test_captured_steps_give_the_plain_logits():
    """Decode steps replayed from captured graphs, requests that join and leave in between (padded batches, slots used
    again), in float32 against the plain implementation: the token before, the states and the windows follow each request."""
    name = "d"
    c = K.CONFIGS[name]
    from nano_vllm_amd.engine.batch import StepEntry
    r = _runner(name, "hip", "float32", 40)
    r.enable_decode_graphs(4, 128, measure_products=False)
    toks = {q: H.random_tokens(c["cfg"].vocab, n, 90 + n) for q, n in (("a", 60), ("b", 41), ("c", 30))}
    got = {q: [] for q in toks}
    pos = {}
    for i in range(200):
        if i == 0 or i == 7 or i == 20:
            q = "abc"[(0, 7, 20).index(i)]
            r.cache.admit(q)
            r.cache.reserve(q, 9)
            got[q].append(r.step([StepEntry(q, toks[q][:9], 0, list(range(9)))]).float().cpu().clone())
            pos[q] = 9
        if not pos:
            break
        entries = []
        for q, p in pos.items():
            r.cache.reserve(q, p + 1)
            entries.append(StepEntry(q, toks[q][p:p + 1], p, [0]))
        out = r.step(entries).float().cpu().clone()
        for row, q in enumerate(list(pos)):
            got[q].append(out[row:row + 1])
            pos[q] += 1
            if pos[q] == len(toks[q]):
                r.cache.release(q)
                del pos[q]
    assert r._graphs
    for q in toks:
        assert K.err(torch.cat(got[q]), K.plain_logits(K.model_folder(name), toks[q])) < MODEL_TOL["float32"], q


@pytest.mark.gpu
def test_trace_replay_of_a_model_folder(tmp_path):
    """bin/trace_run as a process on a Nemidra folder: portions, single tokens and a second request that takes the
    first one's pages."""
    import os
    import subprocess
    import sys
    import numpy as np
    name = "d"
    c = K.CONFIGS[name]
    folder = K.model_folder(name)
    a, b = H.random_tokens(c["cfg"].vocab, 50, 1), H.random_tokens(c["cfg"].vocab, 70, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[33:34], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[34:], "want": [15]}, {"id": "b", "tokens": b[:2], "want": []}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b[2:], "want": [67]}], "end": ["b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                       timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    wa, wb = K.plain_logits(folder, a), K.plain_logits(folder, b)
    vocab = c["cfg"].vocab
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, vocab))
    assert K.err(read(0), wa[[0, 32]]) < MODEL_TOL["float32"]
    assert K.err(read(1), wa[[33]]) < MODEL_TOL["float32"]
    assert K.err(read(2), wa[[49]]) < MODEL_TOL["float32"]
    assert K.err(read(3), wb[[69]]) < MODEL_TOL["float32"]
