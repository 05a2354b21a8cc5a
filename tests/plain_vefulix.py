"""Vefulix written out plainly: whole sequences, no cache, float64, one function per mechanism.

The model is a dictionary of tensors under their checkpoint names and the configuration as the nested dictionary
that `config.json` holds. Nothing here is shared with the engine: it is what the engine is compared with.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, name, eps):
    """Mean taken off, unit standard deviation, weight and bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w[name] + w[name + ".b"]


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ the streams

def read_streams(streams, w, pre):
    """streams [s, T, n] -> what a sublayer reads."""
    return torch.tensordot(w[pre + "in"], streams, dims=1)


def write_streams(streams, y, w, pre):
    """The new streams from the old ones and the sublayer's output y: stream t takes mix[s, t] of every old stream s."""
    new = []
    for t in range(streams.shape[0]):
        x = w[pre + "out"][t] * y
        for s in range(streams.shape[0]):
            x = x + w[pre + "mix"][s, t] * streams[s]
        new.append(x)
    return torch.stack(new)


# ------------------------------------------------------------------ mixers

def soft_gates(h, w, pre, cap):
    """-> (log input gate i, log forget gate f), [T, heads] each."""
    capped = lambda z: cap * torch.tanh(z / cap)
    i = capped(h @ w[pre + "i"].T + w[pre + "i.b"])
    f = torch.nn.functional.logsigmoid(capped(h @ w[pre + "f"].T + w[pre + "f.b"]))
    return i, f


def matrix_memory(q, k, v, i, f):
    """q, k [T, H, D], v [T, H, P], i, f [T, H] -> o [T, H, P]."""
    T, H, D = q.shape
    S, n, m = torch.zeros(H, D, v.shape[-1], dtype=F64), torch.zeros(H, D, dtype=F64), torch.zeros(H, dtype=F64)
    out = []
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + take[:, None] * k[t]
        m = new
        below = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append(torch.stack([S[a].T @ q[t, a] for a in range(H)]) / below[:, None])
    return torch.stack(out)


def mlstm(h, w, pre, m, eps):
    T, H, D, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].T).view(T, H, D)
    v = (h @ w[pre + "v"].T).view(T, H, P)
    o = unit_rms(matrix_memory(q, k, v, *soft_gates(h, w, pre, m["gate_cap"])), eps).reshape(T, H * P)
    return (o * w[pre + "norm"] * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def short_conv(x, taps):
    """x [T, C], taps [C, n]: the last tap multiplies the current token's value, zeros before the start; silu."""
    T, n = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(n):
            src = t - (n - 1) + j
            if src >= 0:
                out[t] += taps[:, j] * x[src]
    return silu(out)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, g):
    """q, k [T, H, D], v [T, H, P], beta, g [T, H] -> o [T, H, P]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    out = []
    for t in range(T):
        row = []
        for a in range(H):
            M = g[t, a] * S[a]
            u = beta[t, a] * (v[t, a] - M.T @ k[t, a])
            M = M + torch.outer(k[t, a], u)
            S[a] = M
            row.append(M.T @ q[t, a])
        out.append(torch.stack(row))
    return torch.stack(out)


def delta(h, w, pre, m, eps):
    T, H, G, D, P = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ w[pre + x].T, w[f"{pre}{x}.conv"]) for x in ("q", "k", "v"))
    shared = torch.arange(H) // (H // G)
    q = unit_vector(q.view(T, G, D))[:, shared] * D ** -0.5
    k = unit_vector(k.view(T, G, D))[:, shared]
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    g = torch.exp(-torch.exp(w[pre + "A_log"]) * torch.nn.functional.softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"]))
    o = unit_rms(delta_rule(q, k, v.view(T, H, P), beta, g), eps) * w[pre + "norm"]
    return (o.reshape(T, H * P) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def latent_attention(h, w, pre, m, eps):
    T, H, D, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = ((unit_rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]) @ w[pre + "uq"].T).view(T, H, D)
    c = unit_rms(h @ w[pre + "dkv"].T, eps) * w[pre + "dkv.norm"]
    k = (c @ w[pre + "uk"].T).view(T, H, D)
    v = (c @ w[pre + "uv"].T).view(T, H, P)
    later = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, H, P, dtype=F64)
    for a in range(H):
        s = ((q[:, a] @ k[:, a].T) * m["scale"]).masked_fill(later, -math.inf)
        sink = w[pre + "sink"][a]
        top = torch.maximum(s.max(-1, keepdim=True).values, sink)
        e = torch.exp(s - top)
        out[:, a] = (e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))) @ v[:, a]
    return out.reshape(T, H * P) @ w[pre + "o"].T


MIXERS = {"mlstm": mlstm, "delta": delta, "latent_attention": latent_attention}


# ------------------------------------------------------------------ feed-forward

def gated_expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def choose_experts(z, top):
    """z: router logits [T, E] -> (ids [T, top], weights [T, top]): the largest logits, a softmax over those alone."""
    values, ids = z.topk(top, -1)
    return ids, torch.softmax(values, -1)


def mixture(h, w, pre, f):
    ids, weights = choose_experts(h @ w[pre + "router"].T + w[pre + "router.b"], f["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t].tolist(), weights[t]):
            out[t] += a * gated_expert(h[t], w, f"{pre}e{e}.")
    if f.get("shared") is not None:
        out = out + gated_expert(h, w, pre + "shared.")
    return out


# ------------------------------------------------------------------ the model

def forward(config, weights, tokens, keep_layers: bool = False):
    """tokens: a list of ids -> logits [T, vocab] (and the sum of the streams after every layer, [layers, T, width])."""
    w = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = layer_norm(w["embed"][torch.as_tensor(tokens, dtype=torch.long)], w, "embed.norm", eps)
    streams, after = torch.stack([x] * config["streams"]), []
    for i, layer in enumerate(config["layers"]):
        pre = f"l{i}."
        h = layer_norm(read_streams(streams, w, pre + "hc1."), w, pre + "norm1", eps)
        streams = write_streams(streams, MIXERS[layer["type"]](h, w, pre + "mix.", layer["mixer"], eps), w, pre + "hc1.")
        if layer.get("mlp") is not None:
            h = layer_norm(read_streams(streams, w, pre + "hc2."), w, pre + "norm2", eps)
            streams = write_streams(streams, mixture(h, w, pre + "mlp.", layer["mlp"]), w, pre + "hc2.")
        after.append(streams.sum(0))
    z = layer_norm(streams.sum(0), w, "final.norm", eps) @ w["head"].T
    cap = config.get("logit_softcap")
    if cap:
        z = cap * torch.tanh(z / cap)
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
