"""Plain, slow implementation of the Bamipel decoder: whole sequences, no cache, no batch.

One function per mechanism, written from the design's equations in this file's own notation.  It
shares no code with the engine: it reads config.json and model.safetensors itself, keeps every
projection as a separate matrix and loops over heads, tokens and keys.  Everything is float64.

The design (r is the residual stream, one row per token):
    r = embed[token]
    per layer:  r <- r + n1b(mixer(n1(r)));  r <- r + n2b(ff(n2(r)))        (ff may be absent)
    n(x) = x / sqrt(mean(x^2) + eps) * w
    logits = head n_final(r)
A layer may run another layer's tensors again.
Rotation: channels (i, i + R/2) of R channels turn by p * f_i, f_i = base^(-2i/R); where the configuration scales
the frequencies, those of long waves are divided by `factor`, those of short waves kept, those between blended.
mixer "latent_attention": cq = n(Wdq h), q = Wuq cq in H heads of [D plain | R rotated]; [c | kr] = Wdkv h, c <- n(c),
    kr (R channels, one for all heads) rotated; per head kp = Wuk c, v = Wuv c;
    s_ij = scale (qp_i.kp_j + qr_i.kr_j), 0 <= i - j < window; softmax; each head's output times sigmoid(Wg h)_head; Wo.
mixer "attention": q = Wq h in H heads of D, k, v in G heads of D and DV; q, k rotated, then each head divided by
    its root mean square; s_ij = scale q_i.k_j, j <= i; softmax; each head's output times sigmoid(Wg h)_head; Wo.
mixer "delta": q = Wq h, k = Wk h in G heads of D, v = Wv h in H heads of DV, each through a causal convolution per
    channel and silu; q <- q / sqrt(sum q^2 + 1e-6) / sqrt(D), k <- k / sqrt(sum k^2 + 1e-6); b = sigmoid(Wb h);
    a = exp(-exp(A_log) softplus(Wa h + dt_bias)) per head; S <- a S; u = b (v - S^T k); S <- S + k u^T; o = S^T q;
    o / sqrt(mean(o^2) + eps) * w * silu(Wg h) per head; Wo.
ff: Wd (max(Wu h, 0)^2).
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


def unit_mean(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def frequencies(rot):
    """f_i of the pairs, with the configuration's scaling of long waves where it has one."""
    R = rot["dims"]
    out = []
    for i in range(R // 2):
        f = rot["base"] ** (-2.0 * i / R)
        sc = rot.get("scaling")
        if sc:
            wave = 2.0 * math.pi / f
            if wave < sc["original"] / sc["high"]:
                pass
            elif wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            else:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def turn_halves(x, rot, first_position=0):
    """x [T, heads, dim]: channels (i, i + R/2) of the first R turned by the token's position."""
    if not rot:
        return x
    half = rot["dims"] // 2
    freqs = frequencies(rot)
    out = x.clone()
    for t in range(x.shape[0]):
        for i in range(half):
            angle = (first_position + t) * freqs[i]
            c, s = math.cos(angle), math.sin(angle)
            u, v = x[t, :, i], x[t, :, i + half]
            out[t, :, i] = u * c - v * s
            out[t, :, i + half] = v * c + u * s
    return out


def softmax_rows(scores):
    e = torch.exp(scores - scores.max())
    return e / e.sum()


def head_gates(h, wg):
    return torch.sigmoid(h @ wg.T)


def latent_parts(cq_raw, low, m, w, p, eps):
    """From the two latents' projections: queries (plain and rotated parts), keys (plain per head, one rotated part) and
    values of every token."""
    T, H, D, R, DV, C = low.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = unit_mean(cq_raw, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).view(T, H, D + R)
    c = unit_mean(low[:, :C], eps) * w[p + "dkv.norm"]
    k_turn = turn_halves(low[:, C:].reshape(T, 1, R), m["rot"])[:, 0]
    return (q[:, :, :D], turn_halves(q[:, :, D:], m["rot"]), (c @ w[p + "uk"].T).view(T, H, D), k_turn,
            (c @ w[p + "uv"].T).view(T, H, DV))


def latent_attend(q_plain, q_turn, k_plain, k_turn, v, scale, window, rows=None):
    """-> [T, H, DV].  rows: the tokens whose output is wanted (default all; the others' stay zero)."""
    T, H = q_plain.shape[0], q_plain.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=v.dtype)
    for head in range(H):
        for i in (range(T) if rows is None else rows):
            lo = 0 if window is None else max(0, i - window + 1)
            s = (k_plain[lo: i + 1, head] @ q_plain[i, head] + k_turn[lo: i + 1] @ q_turn[i, head]) * scale
            out[i, head] = softmax_rows(s) @ v[lo: i + 1, head]
    return out


def latent_attention(h, m, w, p, eps):
    window = m["mask"]["size"] if m.get("mask") else None
    o = latent_attend(*latent_parts(h @ w[p + "dq"].T, h @ w[p + "dkv"].T, m, w, p, eps), m["scale"], window)
    o = o * head_gates(h, w[p + "g"])[:, :, None]
    return o.reshape(h.shape[0], -1) @ w[p + "o"].T


def grouped_attend(q, k, v, scale, rows=None):
    """q [T, H, D], k [T, G, D], v [T, G, DV] -> [T, H, DV], every earlier key and the token's own in sight."""
    T, H = q.shape[0], q.shape[1]
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=v.dtype)
    for head in range(H):
        g = head // per
        for i in (range(T) if rows is None else rows):
            out[i, head] = softmax_rows((k[: i + 1, g] @ q[i, head]) * scale) @ v[: i + 1, g]
    return out


def grouped_attention(h, m, w, p, eps):
    T = h.shape[0]
    q = (h @ w[p + "q"].T).view(T, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T).view(T, m["kv_heads"], m["dim"])
    v = (h @ w[p + "v"].T).view(T, m["kv_heads"], m["vdim"])
    q = unit_mean(turn_halves(q, m.get("rot")), eps)
    k = unit_mean(turn_halves(k, m.get("rot")), eps)
    o = grouped_attend(q, k, v, m["scale"]) * head_gates(h, w[p + "g"])[:, :, None]
    return o.reshape(T, -1) @ w[p + "o"].T


def causal_convolution(x, taps):
    """x [T, channels], taps [channels, n], the last column the token's own."""
    T, n = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(n):
            src = t - (n - 1) + j
            if src >= 0:
                out[t] += taps[:, j] * x[src]
    return out


def delta_step(S, q, k, v, beta, a):
    """One head and token: S [D, DV] -> (S, o)."""
    S = a * S
    u = beta * (v - S.T @ k)
    S = S + torch.outer(k, u)
    return S, S.T @ q


def delta_of_projections(q, k, v, gate, b, z, m, w, p, eps):
    """The rule on the tokens' projections (z: the decays' input before dt_bias) -> [T, H * DV]."""
    T, H, G, D, DV = q.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_convolution(x, w[p + n + ".conv"])) for n, x in (("q", q), ("k", k), ("v", v)))
    q, k, v = q.view(T, G, D), k.view(T, G, D), v.view(T, H, DV)
    q = q / torch.sqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) * D ** -0.5
    k = k / torch.sqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)
    beta = torch.sigmoid(b)
    z = z + w[p + "dt_bias"]
    a = torch.exp(-torch.exp(w[p + "A_log"]) * (torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0)))
    o = torch.zeros(T, H, DV, dtype=v.dtype)
    for head in range(H):
        g = head // (H // G)
        S = torch.zeros(D, DV, dtype=v.dtype)
        for t in range(T):
            S, o[t, head] = delta_step(S, q[t, g], k[t, g], v[t, head], beta[t, head], a[t, head])
    return (unit_mean(o, eps) * w[p + "norm"] * silu(gate).view(T, H, DV)).reshape(T, -1)


def delta_mixer(h, m, w, p, eps):
    q, k, v, gate, b, z = (h @ w[p + n].T for n in ("q", "k", "v", "g", "b", "a"))
    return delta_of_projections(q, k, v, gate, b, z, m, w, p, eps) @ w[p + "o"].T


MIXERS = {"latent_attention": latent_attention, "attention": grouped_attention, "delta": delta_mixer}


def feed_forward(h, w, p):
    return torch.clamp(h @ w[p + "up"].T, min=0).pow(2) @ w[p + "down"].T


def forward(cfg, w, tokens, return_layers=False):
    eps = cfg["norm"]["eps"]
    r = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{layer.get('weights_of', i)}."
        y = MIXERS[layer["type"]](unit_mean(r, eps) * w[p + "norm1"], layer["mixer"], w, p + "mix.", eps)
        r = r + unit_mean(y, eps) * w[p + "norm1b"]
        if layer.get("mlp"):
            y = feed_forward(unit_mean(r, eps) * w[p + "norm2"], w, p + "mlp.")
            r = r + unit_mean(y, eps) * w[p + "norm2b"]
        layers.append(r)
    logits = (unit_mean(r, eps) * w["final.norm"]) @ w["head"].T
    return (logits, torch.stack(layers)) if return_layers else logits


def greedy_generate(cfg, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(forward(cfg, w, tokens)[-1].argmax()))
    return tokens[len(prompt):]
