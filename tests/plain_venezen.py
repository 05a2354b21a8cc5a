"""Venezen written out plainly: whole sequences, no cache, float64, one function per mechanism.

The model is a dictionary of tensors under their checkpoint names and the configuration as the nested dictionary
that `config.json` holds. Nothing here is shared with the engine: it is what the engine is compared with.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def layer_norm(x, weight, eps):
    """Mean taken off, unit standard deviation, a weight, no bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ mixers

def rotate_halves(x, positions, base):
    """x [T, heads, n]: dimension i and dimension i + n/2 turn together by position * base^(-2i/n)."""
    half = x.shape[-1] // 2
    rate = base ** (-torch.arange(half, dtype=F64) / half)
    a = positions.to(F64)[:, None, None] * rate
    u, v = x[..., :half], x[..., half:]
    return torch.cat((u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)), -1)


def latent_attention(h, w, pre, m, eps):
    """Keys and values of every head out of one normed latent per token, beside one rotated key part for all heads."""
    T, H, D, R, P, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    q = (h @ w[pre + "q"].T).view(T, H, D + R)
    q_rot = rotate_halves(q[..., D:], pos, m["rot"]["base"])
    down = h @ w[pre + "dkv"].T
    c = unit_rms(down[:, :rank], eps) * w[pre + "dkv.norm"]
    k_rot = rotate_halves(down[:, None, rank:], pos, m["rot"]["base"])[:, 0]
    k = (c @ w[pre + "uk"].T).view(T, H, D)
    v = (c @ w[pre + "uv"].T).view(T, H, P)
    later = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, H, P, dtype=F64)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"]
        out[:, a] = torch.softmax(s.masked_fill(later, -math.inf), -1) @ v[:, a]
    return out.reshape(T, H * P) @ w[pre + "o"].T


def slopes(heads):
    """What a head takes off a score per token of distance."""
    return [2.0 ** (-8.0 * (a + 1) / heads) for a in range(heads)]


def softmax_plus_one(s):
    """exp(s_j) / (1 + sum exp(s_j)) along the last axis; -inf: not seen."""
    top = s.max(-1, keepdim=True).values.clamp(min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention(h, w, pre, m, eps):
    """Grouped heads whose values are their keys, a distance bias per head, a trailing window, one in the denominator."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[pre + "q"].T).view(T, H, D)
    k = (h @ w[pre + "k"].T).view(T, G, D)
    distance = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = (distance >= 0) & (distance < m["mask"]["size"])
    out = torch.zeros(T, H, D, dtype=F64)
    for a, slope in enumerate(slopes(H)):
        mine = k[:, a // (H // G)]
        s = (q[:, a] @ mine.T) * m["scale"] - slope * distance
        out[:, a] = softmax_plus_one(s.masked_fill(~seen, -math.inf)) @ mine
    return out.reshape(T, H * D) @ w[pre + "o"].T


MIXERS = {"latent_attention": latent_attention, "attention": attention}


# ------------------------------------------------------------------ feed-forward

def dense(h, w, pre):
    lin = lambda x, name: x @ w[pre + name].T + w[pre + name + ".b"]
    return lin(silu(lin(h, "gate")) * lin(h, "up"), "down")


def clamped_expert(h, w, pre, limit):
    g = torch.clamp(h @ w[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ w[pre + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def choose(scores, correction, top, scale):
    """scores [T, E] -> (ids [T, top], weights [T, top]): chosen with the correction, weighed without it."""
    ids = (scores + correction).topk(top, -1).indices
    s = scores.gather(-1, ids)
    return ids, s / (s.sum(-1, keepdim=True) + 1e-20) * scale


def mixture(h, w, pre, f):
    """Routed experts, of which the last `identity` hand their input on, beside one that every token passes."""
    r = f["router"]
    ids, weights = choose(torch.softmax(h @ w[pre + "router"].T, -1), w[pre + "correction"], r["top"], r["scale"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t].tolist(), weights[t]):
            out[t] += a * (h[t] if e >= r["experts"] else clamped_expert(h[t], w, f"{pre}e{e}.", f["expert"]["limit"]))
    if f.get("shared") is not None:
        out = out + clamped_expert(h, w, pre + "shared.", f["shared"]["limit"])
    return out


def feed_forward(h, w, pre, f):
    return dense(h, w, pre) if f["kind"] == "dense" else mixture(h, w, pre, f)


# ------------------------------------------------------------------ the model

def run_order(config):
    """(layer, whether the embedding's output joins the stream in front of it) in the order they run."""
    n, loop = len(config["layers"]), config.get("loop") or {"start": 0, "stop": 0, "times": 1}
    order = [(i, False) for i in range(loop["start"])]
    for k in range(loop["times"]):
        order += [(i, k > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def forward(config, weights, tokens, keep_layers: bool = False):
    """tokens: a list of ids -> logits [T, vocab] (and the stream after every layer run, [runs, T, width])."""
    w = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    start = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    x, after = start, []
    for i, again in run_order(config):
        layer, pre = config["layers"][i], f"l{i}."
        if again:
            x = x + start
        x = x + MIXERS[layer["type"]](layer_norm(x, w[pre + "norm1"], eps), w, pre + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + feed_forward(layer_norm(x, w[pre + "norm2"], eps), w, pre + "mlp.", layer["mlp"])
        after.append(x)
    z = layer_norm(x, w["final.norm"], eps) @ w["embed"].T
    return (z, torch.stack(after)) if keep_layers else z


def read_folder(folder: str):
    """(config.json as a dictionary, the checkpoint's tensors by name) of a model folder."""
    import json
    import os

    from safetensors.torch import load_file

    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    return config, load_file(os.path.join(folder, "model.safetensors"))


def logits(config, weights, tokens):
    return forward(config, weights, tokens)
