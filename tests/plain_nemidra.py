"""Plain, slow implementation of the Nemidra decoder: whole sequences, no cache, no batch.

One function per mechanism, written from the design's equations in this file's own notation.  It
shares no code with the engine: it reads config.json and model.safetensors itself, keeps every
projection as a separate matrix and loops over heads, tokens and keys.  Everything is float64.

The design (r is the residual stream, one row per token):
    e0 = embed[token] + bigram[row] + pos[p];   row = (before * a + token * b) mod B, or B for a first token
    r = e0; the layers in order, some of them several times in a row; every such pass but the first begins
    with r <- r + e0
    per layer:  r <- r + n1b(mixer(n1(r)));  r <- r + n2b(ff(n2(r)))        (ff may be absent)
                r <- r + unit(P (gelu_tanh(G r) * table[token, layer's part])) * w
    n(x) = unit(x) * (1 + w),  unit(x) = x / sqrt(mean(x^2) + eps)
    logits = cap tanh(head n_final(r) / cap)
mixer "parallel": a * left + b * right of the same input.
    left: q in H heads of D, k, v in G heads of D and DV, all with biases; s_ij = scale q_i.k_j, 0 <= i - j < window;
        softmax; output projection with a bias.
    right: per head q (times D^-1/2), k, v, gates i = c tanh((Wi h + bi) / c), f = logsigmoid(c tanh((Wf h + bf) / c));
        m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- likewise with k;  m starts at 0;
        o = S^T q / (max(|n.q|, exp(-m')) + 1e-6);  unit(o) per head, times a weight, times sigmoid(Wg h); projection.
mixer "gla": S <- diag(alpha) S + k v^T, o = S^T q with q times D^-1/2, alpha = sigmoid(A2 A1 h + b)^(1/tau) per key
    channel; unit(o) per head times a weight for all heads, times silu(Wg h); projection.
ff: down(gelu_erf(up h)), or experts: s = softmax(router h); the `top` largest s; sum of scale * s_e * expert_e(h), an
    expert being down(silu(gate h) * (up h)); plus sigmoid(sg h) * shared(h).
"""
from __future__ import annotations

import json
import math
import os

import torch
from safetensors import safe_open


def read_folder(path: str, dtype=torch.float64):
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    weights = {}
    with safe_open(os.path.join(path, "model.safetensors"), "pt", "cpu") as f:
        for name in f.keys():
            t = f.get_tensor(name)
            weights[name] = t.to(dtype) if t.is_floating_point() else t
    return cfg, weights


def unit(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def norm(x, w, eps):
    return unit(x, eps) * (1.0 + w)


def log_sigmoid(z):
    return z.clamp(max=0) - torch.log1p(torch.exp(-z.abs()))


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def bigram_row(cfg, before, token):
    b = cfg["embedding"]["bigram"]
    return b["buckets"] if before is None else (before * b["mul_prev"] + token * b["mul_cur"]) % b["buckets"]


def embed(cfg, w, tokens):
    rows = []
    for p, token in enumerate(tokens):
        row = bigram_row(cfg, tokens[p - 1] if p else None, token)
        rows.append(w["embed"][token] + w["bigram"][row] + w["pos"][p])
    return torch.stack(rows)


def window_attend(q, k, v, scale, window, rows=None):
    """q [T, H, D], k [T, G, D], v [T, G, DV] -> [T, H, DV]; rows: the tokens whose output is wanted."""
    T, H = q.shape[0], q.shape[1]
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=v.dtype)
    for head in range(H):
        g = head // per
        for i in (range(T) if rows is None else rows):
            lo = 0 if window is None else max(0, i - window + 1)
            s = (k[lo: i + 1, g] @ q[i, head]) * scale
            e = torch.exp(s - s.max())
            out[i, head] = (e / e.sum()) @ v[lo: i + 1, g]
    return out


def window_attention(h, m, w, p):
    T = h.shape[0]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, m["kv_heads"], m["dim"])
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, m["kv_heads"], m["vdim"])
    window = m["mask"]["size"] if m.get("mask") else None
    return window_attend(q, k, v, m["scale"], window).reshape(T, -1) @ w[p + "o"].T + w[p + "o.b"]


def matrix_memory_step(S, n, m, q, k, v, i, f):
    """One head and token -> (S, n, m, o)."""
    m_new = max(f + m, i)
    keep, write = math.exp(f + m - m_new), math.exp(i - m_new)
    S = keep * S + write * torch.outer(k, v)
    n = keep * n + write * k
    o = (S.T @ q) / (max(abs(float(n @ q)), math.exp(-m_new)) + 1e-6)
    return S, n, m_new, o


def matrix_memory_of_projections(q, k, v, gate, zi, zf, m, norm_w, eps):
    """q, k [T, H * D], v, gate [T, H * DV], zi, zf [T, H] with their biases -> [T, H * DV]."""
    T, H, D, DV, cap = q.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q, k, v = q.view(T, H, D) * D ** -0.5, k.view(T, H, D), v.view(T, H, DV)
    i, f = cap * torch.tanh(zi / cap), log_sigmoid(cap * torch.tanh(zf / cap))
    o = torch.zeros(T, H, DV, dtype=v.dtype)
    for head in range(H):
        S, n, mm = torch.zeros(D, DV, dtype=v.dtype), torch.zeros(D, dtype=v.dtype), 0.0
        for t in range(T):
            S, n, mm, o[t, head] = matrix_memory_step(S, n, mm, q[t, head], k[t, head], v[t, head], float(i[t, head]),
                                                      float(f[t, head]))
    return unit(o, eps).reshape(T, -1) * norm_w * torch.sigmoid(gate)


def matrix_memory(h, m, w, p, eps):
    q, k, v, gate = (h @ w[p + n].T for n in ("q", "k", "v", "g"))
    zi, zf = (h @ w[p + n].T + w[p + n + ".b"] for n in ("i", "f"))
    return matrix_memory_of_projections(q, k, v, gate, zi, zf, m, w[p + "norm"], eps) @ w[p + "o"].T


def parallel_mixer(h, m, w, p, eps):
    return m["left_scale"] * window_attention(h, m["left"], w, p + "left.") + \
        m["right_scale"] * matrix_memory(h, m["right"], w, p + "right.", eps)


def gla_step(S, q, k, v, alpha):
    S = alpha[:, None] * S + torch.outer(k, v)
    return S, S.T @ q


def gla_of_projections(q, k, v, gate, z, m, norm_w, eps):
    """q, k, z [T, H * D], v, gate [T, H * DV] -> [T, H * DV]."""
    T, H, D, DV = q.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = q.view(T, H, D) * D ** -0.5, k.view(T, H, D), v.view(T, H, DV)
    alpha = torch.exp(log_sigmoid(z) / m["tau"]).view(T, H, D)
    o = torch.zeros(T, H, DV, dtype=v.dtype)
    for head in range(H):
        S = torch.zeros(D, DV, dtype=v.dtype)
        for t in range(T):
            S, o[t, head] = gla_step(S, q[t, head], k[t, head], v[t, head], alpha[t, head])
    return (unit(o, eps) * norm_w * silu(gate).view(T, H, DV)).reshape(T, -1)


def gla_mixer(h, m, w, p, eps):
    q, k, v, gate = (h @ w[p + n].T for n in ("q", "k", "v", "g"))
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return gla_of_projections(q, k, v, gate, z, m, w[p + "norm"], eps) @ w[p + "o"].T


MIXERS = {"parallel": parallel_mixer, "gla": gla_mixer}


def dense(h, w, p):
    return gelu_erf(h @ w[p + "up"].T) @ w[p + "down"].T


def gated_expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(z, router):
    """One token's router logits -> [(expert, weight)]."""
    s = torch.softmax(z, dim=-1)
    order = sorted(range(len(s)), key=lambda e: (-float(s[e]), e))[: router["top"]]
    return [(e, float(s[e]) * router.get("scale", 1.0)) for e in order]


def experts(h, mlp, w, p):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in choose(w[p + "router"] @ h[t], mlp["router"]):
            out[t] += weight * gated_expert(h[t], w, f"{p}e{e}.")
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * gated_expert(h, w, p + "shared.")
    return out


def feed_forward(h, mlp, w, p):
    return dense(h, w, p) if mlp["kind"] == "dense" else experts(h, mlp, w, p)


def token_side(r, tokens, cfg, w, i, eps):
    d = cfg["token_side"]["dim"]
    e = w["side.embed"][torch.as_tensor(tokens, dtype=torch.long), i * d:(i + 1) * d]
    y = (gelu_tanh(r @ w[f"l{i}.side.gate"].T) * e) @ w[f"l{i}.side.proj"].T
    return unit(y, eps) * w[f"l{i}.side.norm"]


def run_order(cfg):
    """[(layer, whether the embedding output is added first)]"""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for turn in range(loop["times"]):
        out += [(i, turn > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def forward(cfg, w, tokens, return_layers=False):
    tokens = [int(t) for t in tokens]
    eps = cfg["norm"]["eps"]
    e0 = embed(cfg, w, tokens)
    r = e0
    layers = []
    for i, again in run_order(cfg):
        if again:
            r = r + e0
        layer, p = cfg["layers"][i], f"l{i}."
        y = MIXERS[layer["type"]](norm(r, w[p + "norm1"], eps), layer["mixer"], w, p + "mix.", eps)
        r = r + norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp"):
            y = feed_forward(norm(r, w[p + "norm2"], eps), layer["mlp"], w, p + "mlp.")
            r = r + norm(y, w[p + "norm2b"], eps)
        r = r + token_side(r, tokens, cfg, w, i, eps)
        layers.append(r)
    logits = norm(r, w["final.norm"], eps) @ w["head"].T
    cap = cfg["logit_softcap"]
    logits = cap * torch.tanh(logits / cap)
    return (logits, torch.stack(layers)) if return_layers else logits


def greedy_generate(cfg, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(forward(cfg, w, tokens)[-1].argmax()))
    return tokens[len(prompt):]
