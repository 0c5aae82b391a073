"""Kaderax, plainly: every mechanism as one slow function in float64, written from the design's equations.

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


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- attention with a bias per distance ---------------------------------------------------------------------------------
def bucket(n, B, D):
    """The row of a table of B rows that a distance n >= 0 reads: its own below B / 2, then logarithmic stretches up to D."""
    half = B // 2
    if n < half:
        return n
    return min(B - 1, half + int(math.floor(math.log(n / half) / math.log(D / half) * (B - half))))


def distance_bias(n, table, D):
    """[n, n, heads]: what position i adds to its score on position j <= i (elsewhere: anything)."""
    row = torch.tensor([bucket(k, table.shape[0], D) for k in range(n)])
    at = torch.arange(n)
    return table[row[torch.clamp(at[:, None] - at[None, :], min=0)]]


def query_temperature(p, temp):
    return 1.0 + temp["coef"] * math.log(math.floor((p + 1) / temp["every"]) + 1)


def biased_attention(h, W, p, m, eps):
    n, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).reshape(n, H, d)
    k = (h @ W[p + "k"].T).reshape(n, G, d)
    v = (h @ W[p + "v"].T).reshape(n, G, dv)
    q = q * torch.tensor([query_temperature(i, m["q_temp"]) for i in range(n)], dtype=F)[:, None, None]
    bias = distance_bias(n, W[p + "rel"], m["bias_max"])
    gate = sigmoid(h @ W[p + "g"].T)
    hidden = torch.ones(n, n, dtype=torch.bool).triu(1)
    out = torch.zeros(n, H, dv, dtype=F)
    for hh in range(H):
        c = hh // (H // G)
        s = m["softcap"] * torch.tanh((q[:, hh] @ k[:, c].T) * m["scale"] / m["softcap"]) + bias[:, :, hh]
        out[:, hh] = gate[:, hh:hh + 1] * (torch.softmax(s.masked_fill(hidden, -math.inf), dim=1) @ v[:, c])
    return out.reshape(n, H * dv) @ W[p + "o"].T


# ---- the decaying linear attention -----------------------------------------------------------------------------------------
def decay_rule(q, k, v, decay, S=None):
    """One head.  q, k [n, d], v [n, dv]: S <- decay S + k v^T, o = S^T q."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=F) if S is None else S.clone()
    o = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o, S


def lightning(h, W, p, m, eps):
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ W[p + "q"].T).reshape(n, H, d)
    k = silu(h @ W[p + "k"].T).reshape(n, H, d)
    v = silu(h @ W[p + "v"].T).reshape(n, H, dv)
    o = torch.zeros(n, H, dv, dtype=F)
    for hh in range(H):
        o[:, hh], _ = decay_rule(q[:, hh], k[:, hh], v[:, hh], m["decay"][hh])
    y = over_rms(o.reshape(n, H * dv), eps) * W[p + "norm"] * sigmoid(h @ W[p + "g"].T)
    return y @ W[p + "o"].T


def parallel(h, W, p, m, eps):
    return m["left_scale"] * biased_attention(h, W, p + "left.", m["left"], eps) \
        + m["right_scale"] * lightning(h, W, p + "right.", m["right"], eps)


# ---- attention through a latent --------------------------------------------------------------------------------------------
def rotate(x, rot):
    """x [n, heads, size] at positions 0 .. n - 1: neighbours 2i and 2i + 1 of the first rot.dims elements turn together."""
    y = x.clone()
    for i in range(rot["dims"] // 2):
        a = torch.arange(x.shape[0], dtype=F) * rot["base"] ** (-2.0 * i / rot["dims"])
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        y[:, :, 2 * i], y[:, :, 2 * i + 1] = u * c - v * s, v * c + u * s
    return y


def softmax_with_sink(s, visible, sink):
    """exp(s) / (exp(sink) + sum exp(s)) along the rows, over the visible entries."""
    s = s.masked_fill(~visible, -math.inf)
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (torch.exp(sink - top) + e.sum(-1, keepdim=True))


def latent_attention(h, W, p, m, eps):
    n, H, dn, dr, dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = over_rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    q = (cq @ W[p + "uq"].T).reshape(n, H, dn + dr)
    down = h @ W[p + "dkv"].T
    c = over_rms(down[:, :R], eps) * W[p + "dkv.norm"]
    k_rot = rotate(down[:, R:].reshape(n, 1, dr), m["rot"])[:, 0]
    q_rot = rotate(q[:, :, dn:], m["rot"])
    k = (c @ W[p + "uk"].T).reshape(n, H, dn)
    v = (c @ W[p + "uv"].T).reshape(n, H, dv)
    visible = torch.ones(n, n, dtype=torch.bool).tril()
    out = torch.zeros(n, H, dv, dtype=F)
    for hh in range(H):
        s = (q[:, hh, :dn] @ k[:, hh].T + q_rot[:, hh] @ k_rot.T) * m["scale"]
        out[:, hh] = softmax_with_sink(s, visible, W[p + "sink"][hh]) @ v[:, hh]
    return (out.reshape(n, H * dv) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def feed_forward(h, W, p):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


MIXERS = {"parallel": parallel, "latent_attention": latent_attention}


def running_order(cfg):
    """[(layer, whether this run begins a pass of the loop)]."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, W, tokens, layers_out=None):
    """Logits [n, vocab] of one sequence."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    start = W["embed"][torch.tensor(list(tokens))]
    x = start.clone()
    for i, enters in running_order(cfg):
        p, layer = f"l{i}.", cfg["layers"][i]
        if enters:
            x = torch.cat([x, start], dim=1) @ W["loop.in"].T
        x = x + mult * MIXERS[layer["type"]](over_rms(x, eps) * W[p + "norm1"], W, p + "mix.", layer["mixer"], eps)
        if layer["mlp"] is not None:
            x = x + mult * feed_forward(over_rms(x, eps) * W[p + "norm2"], W, p + "mlp.")
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
