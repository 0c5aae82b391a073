"""Solulix, plainly: every mechanism as one slow function in float64, written from the design's equations.

Nothing here is shared with the product path.  A sequence is a matrix [n, width] of inputs at positions 0 .. n - 1;
`W` maps tensor names to float64 tensors, `p` is a name prefix ("l3.mix.").
"""
import json
import math
import os

import torch
from safetensors import safe_open

F = torch.float64


def read_folder(folder):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    W = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as f:
        for k in f.keys():
            W[k] = f.get_tensor(k).to(F)
    return cfg, W


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def short_conv(u, w):
    """y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the first row; u [n, channels], w [channels, taps]."""
    n, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(n):
        for j in range(taps):
            at = t - taps + 1 + j
            if at >= 0:
                y[t] += w[:, j] * u[at]
    return y


def seen(n, size, keep_first):
    """[n, n]: whether position i sees position j."""
    m = torch.zeros(n, n, dtype=torch.bool)
    for i in range(n):
        for j in range(i + 1):
            m[i, j] = i - j < size or j < keep_first
    return m


def softmax_plus_one(s, visible):
    """exp(s) / (1 + sum exp(s)) along the last dimension, over the visible entries."""
    s = s.masked_fill(~visible, -math.inf)
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)         # the one in the denominator is a score of zero
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention(h, W, p, m, eps):
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv(h @ W[p + "q"].T, W[p + "q.conv"]).reshape(n, H, d)
    k = short_conv(h @ W[p + "k"].T, W[p + "k.conv"]).reshape(n, G, d)
    v = short_conv(h @ W[p + "v"].T, W[p + "v.conv"]).reshape(n, G, dv)
    visible = seen(n, m["mask"]["size"], m["mask"]["keep_first"])
    out = torch.zeros(n, H, dv, dtype=F)
    for hh in range(H):
        c = hh // (H // G)
        out[:, hh] = softmax_plus_one((q[:, hh] @ k[:, c].T) * m["scale"], visible) @ v[:, c]
    return out.reshape(n, H * dv) @ W[p + "o"].T


def delta_rule(q, k, v, log_g, beta, S=None):
    """One head.  q, k [n, d], v [n, dv], log_g and beta [n]: S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    n, d, dv = q.shape[0], q.shape[1], v.shape[1]
    S = torch.zeros(d, dv, dtype=F) if S is None else S.clone()
    o = torch.zeros(n, dv, dtype=F)
    for t in range(n):
        S = torch.exp(log_g[t]) * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        o[t] = S.T @ q[t]
    return o, S


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta(h, W, p, m, eps):
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(short_conv(h @ W[p + "q"].T, W[p + "q.conv"])).reshape(n, G, d)
    k = silu(short_conv(h @ W[p + "k"].T, W[p + "k.conv"])).reshape(n, G, d)
    v = silu(short_conv(h @ W[p + "v"].T, W[p + "v.conv"])).reshape(n, H, dv)
    q, k = unit(q) * d ** -0.5, unit(k)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    log_g = -torch.exp(W[p + "A_log"]) * torch.nn.functional.softplus(h @ W[p + "a"].T + W[p + "dt_bias"], threshold=1e9)
    o = torch.zeros(n, H, dv, dtype=F)
    for hh in range(H):
        c = hh // (H // G)
        o[:, hh], _ = delta_rule(q[:, c], k[:, c], v[:, hh], log_g[:, hh], beta[:, hh])
    o = over_rms(o, eps) * W[p + "norm"] * silu(h @ W[p + "g"].T).reshape(n, H, dv)
    return o.reshape(n, H * dv) @ W[p + "o"].T


def squared_relu_expert(h, W, p):
    return torch.clamp(h @ W[p + "up"].T, min=0.0) ** 2 @ W[p + "down"].T


def router_choice(h, W, p, r):
    """(chosen outputs of the router [n, top], their weights)."""
    s = torch.softmax(h @ W[p + "router"].T, dim=1)
    order = torch.argsort(-(s + W[p + "correction"]), dim=1, stable=True)[:, :r["top"]]
    w = torch.gather(s, 1, order)
    return order, w / (w.sum(1, keepdim=True) + 1e-20) * r["scale"]


def feed_forward(h, W, p, f):
    if f["kind"] == "dense":
        return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T
    r = f["router"]
    chosen, weight = router_choice(h, W, p, r)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(chosen.shape[1]):
            e = int(chosen[t, j])
            y = h[t:t + 1] if e >= r["experts"] else squared_relu_expert(h[t:t + 1], W, p + f"e{e}.")
            out[t] += weight[t, j] * y[0]
    if f.get("shared"):
        out = out + squared_relu_expert(h, W, p + "shared.")
    return out


MIXERS = {"attention": attention, "delta": delta}


def running_order(cfg):
    """[(layer, pass number if this run begins a pass, else None)]."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, W, tokens, layers_out=None):
    """Logits [n, vocab] of one sequence."""
    eps = cfg["norm"]["eps"]
    start = over_rms(W["embed"][torch.tensor(list(tokens))], eps) * W["embed.norm"]
    x = start.clone()
    for i, turn in running_order(cfg):
        p, layer = f"l{i}.", cfg["layers"][i]
        if turn is not None:
            x = x + W["loop.step"][turn] + (start if turn > 0 else 0.0)
        h = over_rms(x, eps) * W[p + "norm1"]
        y = MIXERS[layer["type"]](h, W, p + "mix.", layer["mixer"], eps)
        if layer["mlp"] is not None:
            y = y + feed_forward(h, W, p + "mlp.", layer["mlp"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return (over_rms(x, eps) * W["final.norm"]) @ W["head"].T


def greedy_generate(cfg, W, prompt, n):
    toks, out = list(prompt), []
    for _ in range(n):
        z = forward(cfg, W, toks)[-1]
        best = int(torch.argmax(z))                      # the smallest id among equals
        toks.append(best)
        out.append(best)
    return out
