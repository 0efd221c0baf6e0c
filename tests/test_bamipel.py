"""Bamipel: every mechanism alone, and the model through the step function and the engine, against
the plain implementation (tests/plain_bamipel.py).  Each test runs on the CPU stand-ins of the
device operations (tests/torch_kernels.py; this checks the stand-ins and the host logic) and, marked
gpu, on the HIP kernels."""
import json

import pytest
import torch

import bamipel_cases as K
import helpers as H
import plain_bamipel as plain
from nano_vllm_amd import LLM, SamplingParams
from nano_vllm_amd.config import BamipelConfig, ConfigError, architecture_of
from nano_vllm_amd.parts import BuildContext, make_part, PartSpec
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
        assert arch.name == "Bamipel"
        again = arch.parse_config(json.loads(json.dumps(d)))
        assert again == c["cfg"].__class__(**{**c["cfg"].__dict__, "dtype": again.dtype}), name
    d = K.CONFIGS["a"]["cfg"].to_dict()
    # what may be left out: the mask, the rotation, its scaling, the feed-forward
    e = json.loads(json.dumps(d))
    e["layers"] = [e["layers"][0], e["layers"][3], e["layers"][6], e["layers"][3]]
    e["layers"][0]["mixer"].pop("mask"), e["layers"][1].pop("mlp")
    e["layers"][3] = json.loads(json.dumps(e["layers"][1]))
    e["layers"][1]["mixer"].pop("rot"), e["layers"][3]["mixer"]["rot"].pop("scaling")
    for l in e["layers"]:
        l.pop("weights_of", None)
    got = BamipelConfig.from_dict(e)
    assert got.layers[0].mixer.window is None and got.layers[1].mixer.rot_dims == 0 and got.layers[1].ff is None
    assert got.layers[3].mixer.rot_scaling is None and got.layers[3].mixer.rot_dims == 8
    # an entry that names an entry without tensors of its own runs what that one runs
    e = json.loads(json.dumps(d))
    e["layers"].append({**e["layers"][2], "weights_of": 2})
    assert BamipelConfig.from_dict(e).layers[7].weights_of == 0
    spec = architecture_of(d).build_spec(K.CONFIGS["a"]["cfg"])
    assert [r.layer for r in spec.order] == [0, 1, 0, 2, 1, 2, 3] and [l.name for l in spec.layers] == ["l0", "l1", "l3", "l6"]

    def broken(change):
        x = json.loads(json.dumps(d))
        change(x)
        with pytest.raises(ConfigError):
            BamipelConfig.from_dict(x)
    broken(lambda x: x["layers"][0].update(type="retention"))
    broken(lambda x: x["layers"][3]["mixer"].update(heads=3))                   # 3 heads on 2 kv heads
    broken(lambda x: x["layers"][1]["mixer"].update(kv_heads=3))
    broken(lambda x: x["layers"][3]["mixer"]["rot"].update(dims=7))
    broken(lambda x: x["layers"][3]["mixer"]["rot"].update(dims=14))            # more than the head
    broken(lambda x: x["layers"][3]["mixer"]["rot"]["scaling"].pop("low"))
    broken(lambda x: x["layers"][3]["mixer"]["rot"]["scaling"].update(low=8.0))  # beyond high
    broken(lambda x: x["layers"][6]["mixer"]["rot"].update(dims=2))             # not the latent layer's rot_dim
    broken(lambda x: x["layers"][6]["mixer"].pop("kv_rank"))
    broken(lambda x: x["layers"][6]["mixer"].pop("q_rank"))
    broken(lambda x: x["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda x: x["layers"][2].update(weights_of=9))
    broken(lambda x: x["layers"][2]["mixer"].update(scale=0.5))                 # differs from its owner
    broken(lambda x: x["layers"][2].update(mlp=None))
    broken(lambda x: x["norm"].update(eps=0.0))
    broken(lambda x: x.pop("vocab"))


def test_the_checkpoint_is_read_by_its_own_names():
    from safetensors import safe_open
    with safe_open(K.model_folder("a") + "/model.safetensors", "pt", "cpu") as f:
        names = set(f.keys())
        shapes = {n: tuple(f.get_slice(n).get_shape()) for n in names}
    common = {"norm1", "norm1b"}
    lat = common | {"mix." + n for n in ("dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv", "g", "o")}
    ff = {"norm2", "norm2b", "mlp.up", "mlp.down"}
    want = {"embed", "head", "final.norm"} | {"l0." + n for n in lat | ff} | {"l6." + n for n in lat}
    want |= {"l1." + n for n in common | ff | {"mix." + x for x in ("q", "k", "v", "q.conv", "k.conv", "v.conv", "b", "a", "A_log", "dt_bias",
                                                                     "norm", "g", "o")}}
    want |= {"l3." + n for n in common | {"mix." + x for x in ("q", "k", "v", "g", "o")}}
    assert names == want, names ^ want
    assert shapes["l0.mix.dq"] == (18, 48) and shapes["l0.mix.uq"] == (48, 18) and shapes["l0.mix.dkv"] == (26, 48)
    assert shapes["l0.mix.g"] == (3, 48) and shapes["l1.mix.g"] == (32, 48) and shapes["l1.mix.a"] == (4, 48)
    assert shapes["l1.mix.k.conv"] == (24, 3) and shapes["l1.mix.norm"] == (8,) and shapes["l3.mix.v"] == (32, 48)
    # rows that pad a packed projection are zero, whatever memory held
    r = _runner("a", "cpu", "float32", 8)
    w = r.model.params["l3.mix.qkv_proj.weight"]
    assert w.shape[0] % 8 == 0 and float(w[4 * 12 + 2 * 12 + 2 * 16 + 4:].abs().sum()) == 0.0


# ------------------------------------------------------------------------------ rotation
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("scaling", [None, (4.0, 1.0, 4.0, 64.0), (8.0, 2.0, 2.0, 40.0), (3.0, 1.0, 32.0, 1000.0)])
def test_frequencies_scaled_by_wavelength(backend, scaling):
    """Short waves kept, long ones divided, those between blended (the three kinds are all there in the first and the
    last case), at positions up to 5000."""
    k, dev = _kernels(backend)
    R, base = 32, 1e4
    rot = {"dims": R, "base": base}
    params = {"head_dim": R, "rotary_dim": R, "theta": base, "max_position": 1 << 30}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
        params["wave_scaling"] = rot["scaling"]
    pe = make_part("position_encoding", PartSpec("rotary_neox", params), BuildContext(k, torch.device(dev), torch.float32, 8, 1 << 30))
    want = plain.frequencies(rot)
    plain_f = plain.frequencies({"dims": R, "base": base})
    if scaling is not None:
        kinds = {("kept" if a == b else "divided" if abs(a * scaling[0] - b) < 1e-12 * b else "blended") for a, b in zip(want, plain_f)}
        assert kinds == ({"kept", "divided"} if scaling[1] == scaling[2] else {"kept", "divided", "blended"})
    for a, b in zip(pe.inv_freq.tolist(), want):
        assert abs(a - b) < 2e-7 * b
    positions = [0, 1, 5, 63, 64, 1000, 5000]
    from types import SimpleNamespace
    table = pe.step_table(SimpleNamespace(positions=torch.tensor(positions, dtype=torch.int32, device=dev), step_cache={})).double().cpu()
    f = torch.tensor(want, dtype=torch.float64)
    for row, p in zip(table, positions):
        assert float((row[:R // 2] - torch.cos(p * f)).abs().max()) < 1e-6 + 3e-7 * p
        assert float((row[R // 2:] - torch.sin(p * f)).abs().max()) < 1e-6 + 3e-7 * p


# ------------------------------------------------------------------------------ preparation of q, k, v
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hq,hkv,D,DV,R,page,pad", [(4, 2, 12, 16, 8, 8, 4), (2, 2, 24, 8, 24, 4, 0), (3, 1, 10, 10, 0, 16, 5), (8, 2, 64, 64, 64, 32, 0)])
def test_heads_divided_by_their_root_mean_square_and_the_gates_columns(backend, dtype, hq, hkv, D, DV, R, page, pad):
    """The rotation comes first in the design and the division after it; rows wider than what they hold; a head of
    tiny numbers, where the eps inside the root counts."""
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(hq * 100 + D)
    positions = [0, 1, 2, 7, 63, 64, 1000, 4000]
    T, eps, base = len(positions), 1e-3, 1e4
    want_width = (hq + hkv) * D + hkv * DV + hq
    x = torch.randn((T, want_width + pad), generator=g) * 2.0
    x[3, :D] *= 0.01
    x[4, hq * D:(hq + 1) * D] *= 0.01
    x = x.to(dtype)
    pos = torch.tensor(positions, dtype=torch.int32, device=dev)
    table = k.rotary_step_table((1.0 / base ** (torch.arange(0, R, 2, dtype=torch.float) / R)).to(dev), pos) if R else None
    slots = torch.tensor([3, 0, 9, 17, 5, -1, 11, 2], dtype=torch.int32, device=dev)
    kc, vc = new_caches(24 // page + 1 if page <= 8 else 2, hkv, D, page, dtype, dev, v_head_dim=DV)
    kc.fill_(float("nan")), vc.fill_(float("nan"))
    gate = torch.full((T, hq), float("nan"), device=dev)
    got_q = k.qk_rownorm_store(x.clone().to(dev), hq, hkv, D, DV, None, None, eps, pos, 0.0, 1, slots, kc, vc, rot_table=table,
                               norm_per_head=True, norm_unit=True, head_gate=gate)
    xd = x.double()
    rot = {"dims": R, "base": base} if R else None
    turned = lambda y: torch.stack([plain.turn_halves(y[t:t + 1], rot, positions[t])[0] for t in range(T)])
    q = plain.unit_mean(turned(xd[:, :hq * D].view(T, hq, D)), eps)
    kk = plain.unit_mean(turned(xd[:, hq * D:(hq + hkv) * D].view(T, hkv, D)), eps)
    v = xd[:, (hq + hkv) * D:(hq + hkv) * D + hkv * DV].view(T, hkv, DV)
    _close(gate, torch.sigmoid(xd[:, want_width - hq:want_width]), torch.float32, "gates")
    vt = vc.shape[4]
    for t in range(T):
        tol = _tol(dtype) + 2.5e-7 * positions[t]
        _close(got_q.reshape(T, hq, D)[t], q[t], dtype, f"q of token {t}", tol=tol)
        s = int(slots[t])
        if s >= 0:
            _close(kc[s // page, :, s % page, :], kk[t], dtype, f"k of token {t}", tol=tol)
            _close(vc[s // page, :, (s % page) // vt, :, (s % page) % vt], v[t], dtype, f"v of token {t}")


# ------------------------------------------------------------------------------ gates per head
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hq,hkv,D,DV,page,lens,q_lens", [
    (4, 2, 12, 16, 8, [30, 9, 41], [1, 1, 41]),               # unequal head sizes: the general kernels
    (3, 1, 10, 10, 16, [50, 33], [17, 33]),
    (8, 2, 64, 64, 32, [130, 70, 100], [1, 2, 64]),           # the matrix cores' kernels in bfloat16
    (4, 4, 128, 128, 64, [700, 1, 150, 200], [1, 1, 1, 130]), # single tokens cut into segments, and one of one key
])
def test_attention_multiplies_every_heads_output_by_its_gate(backend, dtype, hq, hkv, D, DV, page, lens, q_lens):
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(D)
    batch, _, all_slots, pages = K.paged_batch(dev, page, lens, q_lens, 7)
    kc, vc = new_caches(pages, hkv, D, page, dtype, dev, v_head_dim=DV)
    kc.fill_(float("nan")), vc.fill_(float("nan"))
    qs, want = [], []
    T = sum(q_lens)
    gate = torch.rand((T, hq), generator=g)
    gate[0] = 0.0
    at = 0
    for s, (n, c) in enumerate(zip(lens, q_lens)):
        kk, vv, qq = (torch.randn((n, h, d), generator=g).to(dtype) for h, d in ((hkv, D), (hkv, DV), (hq, D)))
        K.fill_cache(kc, vc, all_slots[s], kk, vv)
        qs.append(qq[n - c:].reshape(c, hq * D))
        o = plain.grouped_attend(qq.double(), kk.double(), vv.double(), 0.3, rows=range(n - c, n))[n - c:]
        want.append((o * gate[at:at + c].double()[:, :, None]).reshape(c, hq * DV))
        at += c
    got = k.paged_attention(torch.cat(qs).to(dev), hq, hkv, D, kc, vc, batch, 0, 0.3, None, v_head_dim=DV, head_gate=gate.to(dev))
    k.check_faults()
    _close(got, torch.cat(want), dtype)
    assert float(got[0].abs().max()) == 0.0


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,heads,n_out,k_in", [(1, 3, 20, 10), (37, 2, 7, 16), (16, 4, 64, 32), (70, 5, 130, 176), (8, 6, 128, 384), (600, 20, 128, 72)])
def test_a_product_per_head_times_its_gate(backend, dtype, tokens, heads, n_out, k_in):
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(tokens + n_out)
    x = torch.randn((tokens, heads * k_in), generator=g).to(dtype)
    w = torch.randn((heads * n_out, k_in), generator=g).to(dtype)
    gate = torch.rand((tokens, heads), generator=g)
    y = torch.zeros((tokens, heads * n_out), dtype=dtype, device=dev)
    k.heads_linear(x.to(dev), k_in, w.to(dev), heads, n_out, k_in, False, y, n_out, head_gate=gate.to(dev))
    for h in range(heads):
        want = (x[:, h * k_in:(h + 1) * k_in].double() @ w[h * n_out:(h + 1) * n_out].double().T) * gate[:, h:h + 1].double()
        _close(y[:, h * n_out:(h + 1) * n_out], want, dtype, f"head {h}")


# ------------------------------------------------------------------------------ attention through latents, with a window
def _latent_case(dtype, dev, m, page, lens, q_lens, seed, fav=None, free_passed=False):
    """fav (request, position): that latent row points along a direction of its own, which every query asks for."""
    H_, D, R, DV, Q, C = (m[n] for n in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
    g = torch.Generator().manual_seed(seed)
    window = m["mask"]["size"] if m.get("mask") else None
    batch, _, all_slots, pages = K.paged_batch(dev, page, lens, q_lens, seed, window, free_passed)
    kc, vc = new_caches(pages, 1, C + R, page, dtype, dev, v_head_dim=C)
    kc.fill_(float("nan")), vc.fill_(float("nan"))
    rows = [(torch.randn((n, Q + C + R + H_), generator=g) * 1.5).to(dtype) for n in lens]
    w = {"uq": (torch.randn((H_ * (D + R), Q), generator=g) * 0.4).to(dtype), "uk": (torch.randn((H_ * D, C), generator=g) * 0.4).to(dtype),
         "uv": (torch.randn((H_ * DV, C), generator=g) * 0.4).to(dtype), "dq.norm": (1.0 + 0.3 * torch.randn(Q, generator=g)).to(dtype),
         "dkv.norm": (1.0 + 0.3 * torch.randn(C, generator=g)).to(dtype)}
    if fav is not None:
        s, j = fav
        rows[s][:, :Q + C + R] = 0
        rows[s][:, 0] = 1.0                                  # every query latent along channel 0
        rows[s][:, Q] = 1.0                                  # every key latent along channel 0, the favourite's along 1
        rows[s][j, Q], rows[s][j, Q + 1] = 0.0, 1.0
        for t in (w["uq"], w["uk"]):
            t[:] = 0
        for h in range(H_):
            w["uq"][h * (D + R) + 1, 0] = 4.0
            for i in range(min(D, C)):
                w["uk"][h * D + i, i] = 1.0
        w["dq.norm"][:] = 1.0
        w["dkv.norm"][:] = 1.0
    return batch, all_slots, kc, vc, rows, w


def _plain_latent(rows, w, m, eps, lens, q_lens):
    out = []
    wd = {k: v.double() for k, v in w.items()}
    Q, C, R = m["q_rank"], m["kv_rank"], m["rot_dim"]
    for x, n, c in zip(rows, lens, q_lens):
        x = x.double()
        window = m["mask"]["size"] if m.get("mask") else None
        o = plain.latent_attend(*plain.latent_parts(x[:, :Q], x[:, Q:Q + C + R], m, wd, "", eps), m["scale"], window, rows=range(n - c, n))
        out.append((o * torch.sigmoid(x[:, Q + C + R:])[:, :, None])[n - c:].reshape(c, -1))
    return torch.cat(out)


def _run_latent(k, dev, m, batch, all_slots, kc, vc, rows, w, eps, lens, q_lens):
    """The cache is filled by earlier steps of the same operations, then the step at hand runs."""
    H_, D, R, DV, Q, C = (m[n] for n in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
    inv_freq = (1.0 / (m["rot"]["base"] ** (torch.arange(0, R, 2, dtype=torch.float) / R))).to(dev)
    down = lambda x, pos, slots: k.latent_down(x.to(dev), Q, R, C, H_, w["dq.norm"].to(dev), w["dkv.norm"].to(dev), eps,
                                               k.rotary_step_table(inv_freq, pos), slots, kc, vc, interleaved=False)
    for s, n in enumerate(lens):                                         # the tokens before this step, request by request
        before = n - q_lens[s]
        if before:
            down(rows[s][:before], torch.arange(before, dtype=torch.int32, device=dev),
                 torch.tensor(all_slots[s][:before], dtype=torch.int32, device=dev))
    cq, gate = down(torch.cat([rows[s][lens[s] - q_lens[s]:] for s in range(len(lens))]), batch.positions, batch.groups[0].slot_mapping)
    q, q_head, q2 = k.latent_queries(k.linear(cq, w["uq"].to(dev)), H_, D, R, C, k.rotary_step_table(inv_freq, batch.positions), interleaved=False)
    uk_t = w["uk"].view(H_, D, C).transpose(1, 2).contiguous().view(H_ * C, D).to(dev)
    k.heads_linear(q, q_head, uk_t, H_, C, D, False, q2, C + R)
    window = m["mask"]["size"] if m.get("mask") else None
    o = k.latent_attention(q2, H_, C, R, kc, vc, batch, 0, m["scale"], window=window)
    k.check_faults()
    heads = o.new_empty((o.shape[0], H_ * DV))
    k.heads_linear(o, C, w["uv"].to(dev), H_, DV, C, False, heads, DV, head_gate=gate)
    return heads


def _lat(H_, D, R, DV, Q, C, window, base=1e3, scale=0.2):
    return {"heads": H_, "dim": D, "rot_dim": R, "vdim": DV, "q_rank": Q, "kv_rank": C, "scale": scale, "rot": {"dims": R, "base": base},
            "mask": None if window is None else {"size": window}}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m,page,lens,q_lens", [
    (_lat(3, 10, 6, 14, 18, 20, 10), 8, [30, 9, 41], [1, 1, 41]),                   # single tokens beside a whole prompt
    (_lat(1, 4, 2, 6, 3, 5, 1), 4, [13, 6], [1, 6]),                                # a window of the token itself
    (_lat(4, 32, 32, 32, 64, 64, 48), 32, [130, 70], [2, 70]),                      # the matrix cores' kernels in bfloat16
    (_lat(2, 24, 16, 40, 24, 16, 33), 16, [50, 33], [17, 33]),
    (_lat(2, 64, 16, 32, 48, 176, 70), 64, [200], [37]),                            # key rows of more than 128 entries
    (_lat(2, 16, 32, 16, 40, 96, None), 64, [1, 200], [1, 150]),                    # no window; the first token of a sequence
    (_lat(20, 32, 64, 32, 96, 384, 500, scale=0.05), 64, [1500, 33, 700], [1, 1, 40]),          # shares of a token's window
    (_lat(5, 24, 24, 40, 32, 80, 300), 32, [1000, 2, 640], [1, 1, 50]),             # a key row that ends inside a step of 32 channels
])
def test_attention_through_latents_with_a_window(backend, dtype, m, page, lens, q_lens):
    k, dev = _kernels(backend, dtype)
    if backend == "cpu" and max(lens) > 600 and dtype == torch.bfloat16:
        pytest.skip("the same path as float32 on the stand-ins")
    for free_passed in (False, True):
        batch, all_slots, kc, vc, rows, w = _latent_case(dtype, dev, m, page, lens, q_lens, 5, free_passed=free_passed)
        got = _run_latent(k, dev, m, batch, all_slots, kc, vc, rows, w, 1e-5, lens, q_lens)
        want = _plain_latent(rows, w, m, 1e-5, lens, q_lens)
        _close(got, want, dtype, f"free_passed={free_passed}", tol=1e-4 if dtype == torch.float32 else 4e-2)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page,C,R,window", [(8, 12, 4, 23), (32, 48, 16, 23), (32, 48, 16, 64), (64, 128, 32, 97)])
def test_a_latent_row_just_inside_and_just_outside_the_window(backend, dtype, page, C, R, window):
    """One row takes nearly all the weight of the queries whose window holds it: the last query of a portion, of a whole
    prompt, and a single token follow it at the window's oldest place, and take nothing of it one place further."""
    k, dev = _kernels(backend, dtype)
    m = _lat(2, 16, R, 8, 10, C, window, scale=3.0 / C ** 0.5)
    for n, portion in ((230, 1), (230, 40), (130, 130)):
        for back in (0, window - 1, window):
            batch, all_slots, kc, vc, rows, w = _latent_case(dtype, dev, m, page, [n], [portion], 11, fav=(0, n - 1 - back), free_passed=True)
            got = _run_latent(k, dev, m, batch, all_slots, kc, vc, rows, w, 1e-5, [n], [portion])
            want = _plain_latent(rows, w, m, 1e-5, [n], [portion])
            _close(got, want, dtype, f"{(n, portion, back)}", tol=1e-4 if dtype == torch.float32 else 3e-2)
            flat, peak = w["uv"].float()[:, 0] * C ** 0.5, w["uv"].float()[:, 1] * C ** 0.5
            gate = torch.sigmoid(rows[0][-1, -2:].float()).repeat_interleave(8)
            last = got[-1].float().cpu() / gate
            assert float((last - (peak if back < window else flat)).abs().max()) < 0.12 * float(peak.abs().max()) + 0.05, (n, portion, back)


# ------------------------------------------------------------------------------ rows that come as partial sums
@pytest.mark.gpu
@pytest.mark.parametrize("tokens", [1, 5, 16, 40])
def test_preparations_add_up_a_products_partial_sums(tokens):
    """A product of few rows whose k is split stays as partial sums: the preparation kernels and the activation give
    from them what they give from the finished product."""
    from nano_vllm_amd.kernels.ops import SplitSum
    k, dev = _kernels("hip", torch.bfloat16)
    g = torch.Generator().manual_seed(tokens)
    x = torch.randn((tokens, 1024), generator=g).to(torch.bfloat16).to(dev)
    pos = torch.arange(tokens, dtype=torch.int32, device=dev) * 3
    slots = torch.arange(tokens, dtype=torch.int32, device=dev)
    H_, D, R, Q, C, page = 4, 32, 16, 64, 48, 64
    table = k.rotary_step_table((1.0 / 1e4 ** (torch.arange(0, R, 2, dtype=torch.float) / R)).to(dev), pos)
    mat = lambda n: (torch.randn((n, 1024), generator=g) / 32.0).to(torch.bfloat16).to(dev)
    vec = lambda n: (1 + 0.2 * torch.randn(n, generator=g)).to(torch.bfloat16).to(dev)

    def both(w, run):
        split = k.linear(x, w, deferred=True)
        assert isinstance(split, SplitSum)
        a, b = run(split), run(split.tensor())
        for p, q in zip(a, b):
            assert torch.equal(p, q)
    qw, cw = vec(Q), vec(C)

    def down(low):
        kc, vc = new_caches(1, 1, C + R, page, torch.bfloat16, dev, v_head_dim=C)
        cq, gate = k.latent_down(low, Q, R, C, H_, qw, cw, 1e-5, table, slots, kc, vc, interleaved=False)
        return cq, gate, kc, vc
    both(mat(Q + C + R + H_), down)

    def queries(q):
        rows, step, q2 = k.latent_queries(q, H_, D, R, C, table, interleaved=False)
        return torch.stack([rows[:, h * step:h * step + D] for h in range(H_)]), q2.view(tokens, H_, C + R)[:, :, C:]
    both(mat(H_ * (D + R)), queries)

    def prepare(qkv):
        kc, vc = new_caches(1, 2, D, page, torch.bfloat16, dev)
        gate = torch.empty((tokens, H_), device=dev)
        q = k.qk_rownorm_store(qkv, H_, 2, D, D, None, None, 1e-5, pos, 0.0, 1, slots, kc, vc, rot_table=table, norm_per_head=True,
                               norm_unit=True, head_gate=gate)
        return q.clone(), gate, kc, vc
    both(mat((H_ + 4) * D + 8), prepare)
    for n in (320, 32 * k.cus):               # (a wide weight and few rows: the activation in the product's epilogue)
        w = mat(n)
        for act in ("relu2", "silu"):
            assert torch.equal(k.linear_act(x, w, act), k.act(k.linear(x, w), act)), (n, act)

    def rule(rates):
        shape = (4, 4, 16, 8, 3)
        wt = K.delta_weights(shape, 3, torch.bfloat16)
        proj, _ = K.delta_inputs(shape, tokens, 4, torch.bfloat16)
        states = K.new_states(dev, tokens, shape, 0.5)
        out = k.head_delta(proj.to(dev), rates, 4, 4, 16, 8, 3, wt["conv"].to(dev), wt["dt_bias"].to(dev), wt["A_log"].to(dev),
                           wt["norm"].to(dev), 1e-5, *states, K.state_batch(dev, [1] * tokens, [1] * tokens, list(range(tokens))))
        return out, states[1]
    if tokens <= 16:
        split = k.linear(x, mat(8), out_float32=True, deferred=True)
        assert isinstance(split, SplitSum) and split.dtype == torch.float32 and split.tensor().dtype == torch.float32
        a, b = rule(split), rule(split.tensor())
        for p, q in zip(a, b):
            assert torch.allclose(p.float(), q.float(), rtol=1e-2, atol=1e-5)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,width,inner", [(1, 48, 36), (3, 520, 72), (40, 128, 192), (300, 64, 40)])
def test_the_square_of_relu_after_a_product(backend, dtype, tokens, width, inner):
    k, dev = _kernels(backend, dtype)
    g = torch.Generator().manual_seed(tokens)
    x = torch.randn((tokens, width), generator=g).to(dtype)
    w = (torch.randn((inner, width), generator=g) / width ** 0.5).to(dtype)
    got = k.linear_act(x.to(dev), w.to(dev), "relu2")
    _close(got, torch.clamp(x.double() @ w.double().T, min=0).pow(2), dtype)


# ------------------------------------------------------------------------------ the delta rule
DELTA_SHAPES = [(4, 2, 12, 8, 3), (2, 2, 10, 14, 1), (3, 1, 5, 7, 5), (2, 1, 40, 70, 2), (2, 2, 64, 64, 4), (2, 1, 128, 128, 4),
                (1, 1, 130, 20, 2)]          # heads, kv_heads, dim, vdim, taps


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", DELTA_SHAPES)
def test_the_delta_rule_in_portions_of_every_size_and_token_by_token(backend, dtype, shape):
    """One request: whole, token by token, and in portions down to two tokens and shorter than the convolution, on a
    slot that held NaN (a request's start reads nothing of what its slot held)."""
    k, dev = _kernels(backend, dtype)
    T, eps = 45, 1e-5
    w = K.delta_weights(shape, 11, dtype)
    inputs = K.delta_inputs(shape, T, 12, dtype)
    want = K.plain_delta(shape, w, inputs, eps)
    cuttings = ([T], [1] * T, [2, 2, 1, 3, 1, 1, 2, 17, 5, 2, 9], [1, 44], [44, 1], [13, 2, 30])
    for portions in cuttings[:3] if backend == "cpu" and shape[2] >= 64 else cuttings:
        states = K.new_states(dev, 3, shape)
        outs, pos = [], 0
        for n in portions:
            outs.append(K.run_delta(k, dev, shape, w, tuple(t[pos:pos + n] for t in inputs), eps, states, [n], [pos], [1]))
            pos += n
        _close(torch.cat(outs), want, dtype, portions[:4], 4e-2 if dtype == torch.bfloat16 else 1e-4)
        assert torch.isnan(states[1][0]).all() and torch.isnan(states[1][2]).all(), "another request's slot was written"


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_delta_rule_of_unequal_requests_in_one_batch(backend):
    """Steps of requests of unequal lengths (single tokens first, as the batch orders them), on slots in another order
    than the requests; one request ends and another takes its slot."""
    k, dev = _kernels(backend)
    shape, eps = (4, 2, 12, 8, 3), 1e-6
    w = K.delta_weights(shape, 21, torch.float32)
    lens = {"a": 30, "b": 3, "c": 55, "d": 17, "e": 26}
    inputs = {r: K.delta_inputs(shape, n, 30 + i, torch.float32) for i, (r, n) in enumerate(lens.items())}
    want = {r: K.plain_delta(shape, w, inputs[r], eps) for r in lens}
    states = K.new_states(dev, 4, shape)
    slot = {"a": 2, "b": 0, "c": 3, "d": 1, "e": 0}
    steps = [[("b", 0, 1), ("a", 0, 30), ("c", 0, 20), ("d", 0, 2)],
             [("b", 1, 1), ("d", 2, 1), ("c", 20, 33)],
             [("b", 2, 1), ("c", 53, 1), ("d", 3, 14)],
             [("c", 54, 1), ("e", 0, 26)]]                              # e takes b's slot, which holds b's last state
    got = {r: [] for r in lens}
    for step in steps:
        part = tuple(torch.cat([inputs[r][i][s:s + n] for r, s, n in step]) for i in range(2))
        out = K.run_delta(k, dev, shape, w, part, eps, states, [n for _, _, n in step], [s for _, s, _ in step],
                          [slot[r] for r, _, _ in step])
        row = 0
        for r, s, n in step:
            got[r].append(out[row:row + n])
            row += n
    for r in lens:
        _close(torch.cat(got[r]), want[r], torch.float32, r, 1e-4)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dim", [16, 64])
def test_the_delta_rule_keeps_and_forgets_by_its_decay(backend, dim):
    """A head whose decay is next to one still reads out, hundreds of tokens later, the value written for a key that
    no later key touched, and reads its own token's write; a head that forgets fast does not.  The state is float32."""
    k, dev = _kernels(backend)
    shape, eps, T = (2, 1, dim, 8, 1), 1e-6, 400
    heads, kv_heads, dim, vdim, taps = shape
    w = K.delta_weights(shape, 5, torch.float32, slow=0)
    w["A_log"][1] = 1.0
    w["conv"][:] = 1.0                                       # one tap of weight 1: the convolution passes its input
    C = 2 * dim + heads * vdim
    proj = torch.zeros((T, C + heads * vdim))
    proj[:, :2 * dim] = -30.0                                # silu(-30) ~ 0; unit norm makes q and k axis vectors
    proj[0, dim + 3] = 30.0                                  # token 0 writes at key axis 3
    proj[1:, dim + 5] = 30.0                                 # every later token writes at key axis 5
    proj[-1, 3] = 30.0                                       # the last token asks for axis 3
    proj[:-1, 5] = 30.0                                      # the others for axis 5: what they write themselves
    g = torch.Generator().manual_seed(9)
    proj[:, 2 * dim:C] = torch.randn((T, heads * vdim), generator=g)
    proj[:, C:] = 2.0
    rates = torch.zeros((T, 2 * heads))
    rates[:, :heads] = 30.0                                  # beta = 1: a write replaces what its key read
    w["norm"][:] = 1.0
    w["dt_bias"][:] = 0.0
    inputs = (proj, rates)
    want = K.plain_delta(shape, w, inputs, eps)
    own = torch.nn.functional.silu(proj[10, 2 * dim:C]).double()
    assert float((want[10, :vdim] / want[10, :vdim].norm() - own[:vdim] / own[:vdim].norm()).abs().max()) < 1e-4
    for portions in ([T], [T - 1, 1], [150, 249, 1]):
        states = K.new_states(dev, 1, shape)
        outs, pos = [], 0
        for n in portions:
            outs.append(K.run_delta(k, dev, shape, w, tuple(t[pos:pos + n] for t in inputs), eps, states, [n], [pos], [0]))
            pos += n
        got = torch.cat(outs).cpu()
        _close(got, want, torch.float32, portions, 1e-4)
        first = torch.nn.functional.silu(proj[0, 2 * dim:2 * dim + vdim])
        assert float((got[-1, :vdim] / got[-1, :vdim].norm() - first / first.norm()).abs().max()) < 1e-3, "the far write is lost"


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 4])
def test_an_impulse_shows_for_exactly_the_convolutions_taps(backend, dtype, taps):
    """A value projection that is nonzero at one token only: the state takes writes at that token and the taps - 1 after
    it, whole and with a portion's edge inside the convolution."""
    k, dev = _kernels(backend, dtype)
    shape, T, at = (1, 1, 8, 8, taps), 20, 9
    w = K.delta_weights(shape, 3, dtype)
    proj, rates = K.delta_inputs(shape, T, 4, dtype)
    proj[:, 16:24] = 0
    proj[at, 16:24] = 3.0
    proj[:, 24:] = 5.0
    rates[:, 1] = 100.0                                       # the decay is next to nothing: what is read is the token's own write
    for portions in ([T], [at + 1, T - at - 1], [1] * T):
        states, outs, pos = K.new_states(dev, 1, shape), [], 0
        for n in portions:
            outs.append(K.run_delta(k, dev, shape, w, (proj[pos:pos + n], rates[pos:pos + n]), 1e-3, states, [n], [pos], [0]))
            pos += n
        seen = torch.cat(outs).float().cpu().abs().amax(-1) > 1e-4
        assert seen.nonzero().flatten().tolist() == list(range(at, at + taps)), portions


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(4, 2, 12, 8, 3), (2, 2, 64, 64, 4), (1, 1, 130, 20, 6), (3, 1, 30, 18, 1), (2, 1, 128, 128, 4)])
def test_long_portions_beside_single_tokens(backend, dtype, shape):
    """Portions of more than a block of 64 tokens (and of exactly one, one more, and a few tokens) beside single tokens,
    from a start and from a state: outputs and states are the plain implementation's, whatever runs them."""
    k, dev = _kernels(backend, dtype)
    if backend == "cpu" and (dtype == torch.bfloat16 or shape[2] > 64):
        pytest.skip("the stand-ins run one way only")
    heads, kv_heads, dim, vdim, taps = shape
    eps = 1e-5
    w = K.delta_weights(shape, 41, dtype)
    lens = {"a": 9, "b": 130, "c": 67, "d": 200, "e": 68}
    inputs = {r: K.delta_inputs(shape, n, 50 + i, dtype) for i, (r, n) in enumerate(lens.items())}
    want = {r: K.plain_delta(shape, w, inputs[r], eps) for r in lens}
    slot = {"a": 2, "b": 0, "c": 4, "d": 1, "e": 3}
    steps = [[("a", 0, 8), ("b", 0, 64), ("c", 0, 65), ("d", 0, 3)],
             [("a", 8, 1), ("b", 64, 1), ("d", 3, 131), ("c", 65, 2), ("e", 0, 67)],
             [("e", 67, 1), ("b", 65, 65), ("d", 134, 66)]]
    found = {}
    ways = [(True, True), (False, False)] if backend == "hip" else [(True, True)]
    for blocks, single in ways:
        if backend == "hip":
            k.delta_blocks, k.delta_single_kernel = blocks, single
        try:
            states, got = K.new_states(dev, 6, shape), {r: [] for r in lens}
            for step in steps:
                part = tuple(torch.cat([inputs[r][i][s:s + n] for r, s, n in step]) for i in range(2))
                out = K.run_delta(k, dev, shape, w, part, eps, states, [n for _, _, n in step], [s for _, s, _ in step], [slot[r] for r, _, _ in step])
                row = 0
                for r, s, n in step:
                    got[r].append(out[row:row + n])
                    row += n
            for r in lens:
                _close(torch.cat(got[r]), want[r], dtype, (r, blocks), 4e-2 if dtype == torch.bfloat16 else 1e-4)
            assert torch.isnan(states[1][5]).all()
            found[blocks] = states
        finally:
            if backend == "hip":
                k.delta_blocks = k.delta_single_kernel = True
    if backend == "hip":
        # the states agree far below what bfloat16's outputs show (the inputs are the same numbers)
        assert torch.equal(found[True][0][:5], found[False][0][:5])
        _close(found[True][1][:5], found[False][1][:5].cpu(), torch.float32, "states")


@pytest.mark.parametrize("backend", BACKENDS)
def test_blocks_of_keys_that_are_nearly_one_direction(backend):
    """Keys that all lie within a few degrees, full write strengths and next to no decay: every write cancels most of what
    the ones before it left, which is where a block's triangular system is hardest."""
    k, dev = _kernels(backend)
    shape, T, eps = (2, 1, 32, 16, 1), 150, 1e-6
    w = K.delta_weights(shape, 8, torch.float32)
    w["A_log"][:] = -9.0
    w["conv"][:] = 1.0
    proj, rates = K.delta_inputs(shape, T, 9, torch.float32)
    proj[:, 32:64] = 3.0 + 0.1 * proj[:, 32:64]
    rates[:, :2] = 8.0
    want = K.plain_delta(shape, w, (proj, rates), eps)
    states = K.new_states(dev, 1, shape)
    _close(K.run_delta(k, dev, shape, w, (proj, rates), eps, states, [T], [0], [0]), want, torch.float32, "one direction", 2e-4)


def test_portions_are_cut_into_blocks():
    from nano_vllm_amd.kernels.ops import delta_blocks
    units, chains = delta_blocks([1, 1, 130, 2, 64], 2)
    assert units == [2, 2, 64, 0, 2, 66, 64, 0, 2, 130, 2, 0, 3, 132, 2, 0, 4, 134, 64, 0]
    assert chains == [0, 3, 2, 0, 3, 1, 3, 0, 4, 1, 4, 0]


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
    n = 70 if (backend, name) == ("cpu", "b") else 110
    toks = H.random_tokens(c["cfg"].vocab, n, 1)
    want = K.plain_logits(K.model_folder(name), toks)
    r = _runner(name, backend, "float32", 40)
    windows = {l.mixer.window if l.kind == "latent_attention" else None for l in c["cfg"].layers if l.kind != "delta"}
    assert len(r.cache.groups) == len(windows)
    assert len(r.layer_caches) == len(c["cfg"].layers)          # a layer that runs another's tensors has a cache of its own
    for portions in (H.whole(n), H.last_one_by_one(n, 45), H.changing_portions(n, 2), [1] * 3 + [2] * 10 + [n - 23]):
        got = H.run_portions(r, "x", toks, portions)
        assert K.err(got, want) < MODEL_TOL["float32"], portions
    assert all(pool.num_free == 40 for pool in r.cache.pools)


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["a", "b", "d"])
def test_bfloat16_follows_the_plain_logits_under_every_cutting(name):
    c = K.CONFIGS[name]
    n = 130
    toks = H.random_tokens(c["cfg"].vocab, n, 3)
    want = K.plain_logits(K.model_folder(name, "bfloat16"), toks)
    r = _runner(name, "hip", "bfloat16", 40)
    for portions in (H.whole(n), H.last_one_by_one(n, 40), H.changing_portions(n, 4)):
        e = K.errors(H.run_portions(r, "x", toks, portions), want)
        assert float(e.median()) < 0.05 and float(e.max()) < 0.3, (portions, float(e.median()), float(e.max()))


@pytest.mark.gpu
def test_a_larger_model_over_long_prompts():
    """Six hundred tokens through a model with windows over several pages and key rows of 128 entries and more:
    whole, in changing portions, and its last tokens one by one."""
    name = "e"
    c = K.CONFIGS[name]
    n = 600
    toks = H.random_tokens(c["cfg"].vocab, n, 17)
    want = K.plain_logits(K.model_folder(name), toks)
    r = _runner(name, "hip", "float32", 12)
    assert len(r.cache.groups) == 3
    for portions in (H.whole(n), H.changing_portions(n, 5), H.last_one_by_one(n, 180)):
        assert K.err(H.run_portions(r, "x", toks, portions), want) < MODEL_TOL["float32"], portions[:4]
    assert all(pool.num_free == 12 for pool in r.cache.pools)
    want16 = K.plain_logits(K.model_folder(name, "bfloat16"), toks)
    r = _runner(name, "hip", "bfloat16", 12)
    for portions in (H.whole(n), H.changing_portions(n, 5), H.last_one_by_one(n, 60)):
        e = K.errors(H.run_portions(r, "x", toks, portions), want16)
        assert float(e.median()) < 0.05 and float(e.max()) < 0.3, (portions[:4], float(e.median()), float(e.max()))


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
    # 171 tokens one by one: every window passes over decoded tokens, the grouped attention sees them all
    c = K.CONFIGS[name]
    n = 171
    toks = H.random_tokens(c["cfg"].vocab, n, 5)
    want = K.plain_logits(K.model_folder(name), toks)
    r = _runner(name, backend, "float32", 48)
    assert K.err(H.run_portions(r, "x", toks, [1] * n), want) < MODEL_TOL["float32"]
    if name == "a":
        # a window's group holds the pages of its window only, the grouped attention's group all of them
        r.cache.admit("y")
        for pos in range(n):
            r.cache.reserve("y", pos + 1)
        by_window = {g.window: sum(1 for p in t if p >= 0) for g, t in zip(r.cache.groups, r.cache.requests["y"].tables)}
        assert by_window[10] <= 3 and by_window[21] <= 4 and by_window[None] == 22, by_window
        r.cache.release("y")


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
        assert K.err(got[rid], one) < 2e-5, rid


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_residual_stream_after_every_layer(backend):
    """Layer by layer: the float32 stream after a layer is the plain implementation's.  The stream takes a layer's
    last addend inside the norm that follows, so it is read where that norm leaves it."""
    name = "a"
    c = K.CONFIGS[name]
    toks = H.random_tokens(c["cfg"].vocab, 37, 9)
    cfg, w = K.plain_model(K.model_folder(name))
    _, streams = plain.forward(cfg, w, toks, return_layers=True)
    r = _runner(name, backend, "float32", 8)
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
    at, ends = 0, []
    for layer in cfg["layers"]:
        at += 2 if layer.get("mlp") else 1
        ends.append(at)                                   # the norm that first sees the stream after this layer
    assert len(seen) == at + 1
    for i, want in enumerate(streams):
        assert float((seen[ends[i]].double() - want).abs().max() / want.abs().max()) < 3e-5, i


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
        assert o["token_ids"] == plain.greedy_generate(cfg, w, p, 10), len(p)
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
def test_trace_replay_of_a_model_folder(tmp_path):
    """bin/trace_run as a process on a Bamipel folder: portions, single tokens and a second request that takes the
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
