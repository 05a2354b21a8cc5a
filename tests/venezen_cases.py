"""Test configurations of the Venezen design, all the tests' own, and their plain evaluation (tests/plain_venezen.py).

The configurations differ from each other in every size: both mixers in several orders, loops that begin at the first layer,
end at the last, hold one layer or several, run once to three times, and no loop; layers without a feed-forward, experts with
and without identity ones and a shared one, one expert per token and all of them, sizes that are no whole steps of 8, single
heads, head counts that are no powers of two, windows of one token up to beyond every request. `make_folder` draws weights whose
rows have unit size on unit inputs, so that sublayers matter beside the stream, score scales are large, so that the softmax is
peaked and a key that is wrongly seen or missed moves the logits, and biases, corrections and routers are scaled up so that
leaving one out moves them far beyond the tolerance.
"""
from __future__ import annotations

import os

import torch

import plain_venezen
from cut_cases import Cuts
from helpers import Driver, random_ids, rel_err
from mini_engine_amd.config.model_config import VenezenConfig
from mini_engine_amd.parts.block import settled
from mini_engine_amd.parts.base import Settled
from mini_engine_amd.weights.random_init import write_random_model


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=1e4):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                                                  "scale": scale, "rot": {"dims": rot_dim, "base": base}}}


def _attention(heads, kv_heads, dim, window, scale):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": window}}}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, identity, top, limit, scale=1.5, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "identity": identity, "top": top, "scale": scale}}
    if shared:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    return mlp


def _with(layer, mlp):
    return dict(layer, mlp=mlp)


def _model(vocab, width, eps, scale, layers, loop=None):
    d = {"architecture": "Venezen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def _real(moe):
    return [_with(_latent(16, 128, 64, 128, 192, 192 ** -0.5 * 1.5, 1e6), _dense(3072)), _with(_attention(16, 8, 128, 200, 128 ** -0.5 * 2), moe),
            _with(_latent(16, 128, 32, 64, 96, 128 ** -0.5 * 2, 1e4), moe), _with(_attention(16, 16, 64, 130, 64 ** -0.5 * 2), moe)]


CONFIGS = {
    "mix": _model(103, 48, 1e-5, 3.0, [
        _with(_latent(3, 16, 8, 24, 40, 0.7), _dense(56)),
        _with(_attention(4, 2, 16, 21, 0.8), _moe(24, 6, 2, 3, 1.2, 1.5, (40, 0.9))),
        _with(_latent(2, 24, 16, 8, 32, 0.6, 500.0), _moe(16, 5, 3, 2, 0.8, 0.7)),
        _with(_attention(6, 3, 8, 40, 1.0), None),
    ], (1, 3, 2)),
    # sizes in no whole steps of 8; the loop begins at the first layer and runs three times; no identity experts, one per token
    "odd": _model(97, 36, 1e-6, 1.3, [
        _with(_attention(3, 1, 10, 7, 1.1), None),
        _with(_latent(5, 12, 6, 10, 22, 0.9), _dense(20)),
        _with(_attention(5, 5, 14, 3, 0.9), _moe(12, 5, 0, 1, 1.5, 2.0, (11, 2.0))),
        _with(_latent(1, 10, 2, 14, 18, 1.0), _moe(9, 3, 4, 5, 0.7, 1.0)),
    ], (0, 2, 3)),
    # what a model may make equal or one: one head, one pass, one expert, a window of one token, a scale of one
    "one": _model(64, 32, 1e-5, 1.0, [
        _with(_latent(1, 16, 16, 16, 16, 1.0), _moe(16, 1, 1, 1, 1.0, 1.0, (16, 1.0))),
        _with(_attention(1, 1, 16, 1, 1.0), _dense(32)),
        _with(_attention(2, 2, 16, 16, 1.2), _moe(16, 2, 0, 1, 1.0, 1.0)),
    ], (0, 3, 1)),
    # a loop of one layer that ends the model; every expert chosen; head sizes 48 and 32 in kernels of whole steps of 16; a width in
    # whole 16-byte pieces around sizes that are not
    "mid": _model(120, 64, 1e-5, 5.0, [
        _with(_attention(8, 2, 40, 33, 0.6), _moe(24, 2, 1, 3, 1.4, 2.5, (28, 1.1))),
        _with(_latent(7, 20, 10, 12, 26, 0.8, 2e4), _dense(72)),
        _with(_attention(2, 1, 24, 64, 0.9), _moe(16, 9, 3, 4, 0.9)),
    ], (2, 3, 3)),
    # latent layers alone: every token stays visible, no window; no loop
    "pages": _model(70, 40, 1e-5, 2.0, [
        _with(_latent(2, 16, 4, 8, 24, 1.0), _moe(16, 4, 2, 2, 1.0)),
        _with(_latent(4, 8, 8, 16, 32, 1.1, 100.0), _moe(24, 3, 1, 1, 1.3, 1.2, (16, 1.5))),
    ]),
    # windows alone: pages behind the longest one are given back; the whole model runs twice
    "windows": _model(50, 24, 1e-5, 2.0, [
        _with(_attention(2, 2, 8, 24, 1.3), _moe(16, 4, 1, 2, 1.0)),
        _with(_attention(3, 3, 12, 5, 1.0), None),
    ], (0, 2, 2)),
    # the layer sizes of a real model (GPU only); every token takes all 6, so that no choice can fall otherwise in bfloat16 than in
    # float32 and every row can be held to the tolerance
    "real": _model(2048, 1024, 1e-6, 4.0, _real(_moe(384, 4, 2, 6, 2.0, 2.0, (1536, 3.0))), (1, 3, 2)),
    # the same with 4 of 24 per token: a token whose choice hangs on two close scores may choose otherwise in bfloat16, so these rows
    # are held to the tolerance in the mean
    "routed": _model(2048, 1024, 1e-6, 4.0, _real(_moe(384, 16, 8, 4, 2.0, 2.0, (1536, 3.0))), (1, 3, 2)),
}
SEEDS = {"mix": 51, "odd": 52, "one": 53, "mid": 54, "pages": 55, "windows": 56, "real": 57, "routed": 58}
PAGE = {"mix": 16, "odd": 8, "one": 4, "mid": 32, "pages": 16, "windows": 8, "real": 16, "routed": 16}
SMALL = ("mix", "odd", "one", "mid", "pages", "windows")


def _every_expert(config):
    """The configuration with every expert chosen by every token: no choice can then fall otherwise in bfloat16 than in float32."""
    def all_of(f):
        return dict(f, router=dict(f["router"], top=f["router"]["experts"] + f["router"]["identity"]))
    return dict(config, layers=[dict(l, mlp=all_of(l["mlp"])) if l["mlp"] is not None and l["mlp"]["kind"] == "moe" else l for l in config["layers"]])


for _name in SMALL:
    CONFIGS[_name + "-all"], SEEDS[_name + "-all"], PAGE[_name + "-all"] = _every_expert(CONFIGS[_name]), SEEDS[_name], PAGE[_name]


def make_folder(name: str, path: str) -> str:
    """A checkpoint of the configuration with seeded random weights in bfloat16, reshaped so that every mechanism shows (see
    the module's text)."""
    from safetensors import safe_open
    from safetensors.torch import save_file

    cfg = VenezenConfig.from_dict(CONFIGS[name])
    write_random_model(cfg, SEEDS[name], path, torch.bfloat16)
    file = os.path.join(path, "model.safetensors")
    with safe_open(file, "pt", device="cpu") as f:
        tensors = {k: f.get_tensor(k) for k in f.keys()}
    for k in tensors:
        t = tensors[k].float()
        if k.endswith(".b"):
            t = t * 40.0
        elif k.endswith(".correction"):
            t = t * 10.0
        elif k == "embed":
            t = t * 50.0
        elif t.dim() == 2:
            t = t / (0.02 * t.shape[1] ** 0.5)                         # unit outputs on unit inputs
            if k.endswith(".router"):
                t = t * 1.5
        tensors[k] = t.to(tensors[k].dtype)
    save_file(tensors, file, metadata={"format": "pt"})
    return path


_plain: dict = {}


def plain_model(folder: str):
    if folder not in _plain:
        _plain[folder] = plain_venezen.read_folder(folder)
    return _plain[folder]


def plain_logits(folder: str, ids: list) -> torch.Tensor:
    key = (folder, tuple(ids))
    if key not in _plain:
        cfg, w = plain_model(folder)
        _plain[key] = plain_venezen.logits(cfg, w, ids)
    return _plain[key]


CUTS = Cuts(CONFIGS, PAGE, plain_logits)


def stream_behind(h, residual):
    """The stream with what a layer has left to be added, float32."""
    h, residual = settled(h, residual)
    if isinstance(h, Settled):
        return residual
    return residual + (h.float().sum(0) if h.dim() == 3 else h.float())


def layers_one_by_one(env, name):
    """The stream after every layer run, float32, against the plain evaluation's."""
    runner, manager, folder = env.runner(name, 4 * -(-19 // PAGE[name]), 1)
    ids = random_ids(19, CONFIGS[name]["vocab"], 77)
    cfg, w = plain_model(folder)
    _, want = plain_venezen.forward(cfg, w, ids, keep_layers=True)
    got, inner = [], runner.model.layers
    kept = [layer.forward for layer in inner]

    def spy(forward):
        def run(*a):
            h, residual = forward(*a)
            got.append(stream_behind(h, residual))
            return h, residual
        return run

    try:
        for layer in inner:
            layer.forward = spy(layer.forward)
        Driver(runner, manager).step({"r": ids}, end=["r"])
    finally:
        for layer, forward in zip(inner, kept):
            layer.forward = forward
    order = plain_venezen.run_order(cfg)
    assert len(got) == len(want) == len(order)
    for i, (a, b) in enumerate(zip(got, want)):
        assert a.dtype == torch.float32 and rel_err(a, b) <= env.tol, f"{name}: run {i} (layer {order[i][0]}): {rel_err(a, b):.3g}"


def real_sizes(env_f32, env_bf16, name="real", every_row=True):
    """At the layer sizes of a real model: float32 against the plain evaluation on a short prompt; then a prompt of 600
    tokens whole, in portions and with its last tokens decoded, bfloat16 against float32 of the same engine: every row
    within the tolerance, or (a model whose tokens choose among experts) the rows in the mean and the median."""
    page, V = PAGE[name], CONFIGS[name]["vocab"]
    short = random_ids(40, V, 900)
    runner, manager, folder = env_f32.runner(name, 8, 1)
    d = Driver(runner, manager)
    d.step({"s": short[:33]})
    d.step({"s": short[33:34]})
    d.step({"s": short[34:]}, end=["s"])
    CUTS.check(env_f32, folder, short, d.result("s"), f"{name} short prompt in float32")
    n = 600
    ids = random_ids(n, V, 901)
    got = {}
    for env in (env_f32, env_bf16):
        runner, manager, folder = env.runner(name, 2 * -(-n // page), 2)
        d = Driver(runner, manager)
        d.step({"w": ids})
        d.step({"r": ids[:300]})
        d.step({"r": ids[300:302]})
        d.step({"r": ids[302:580]})
        for t in range(580, n):
            d.step({"r": ids[t:t + 1]})
        got[env.dtype] = (d.result("w"), d.result("r"))
    (wf, rf), (wb, rb) = got[torch.float32], got[torch.bfloat16]
    assert rel_err(rf, wf.double().cpu()) <= 1e-4, "float32: the cut request differs from the whole one"
    wide = wf.double().cpu()
    for got_b, what in ((wb, "whole"), (rb, "cut")):
        if every_row:
            assert rel_err(got_b, wide) <= env_bf16.tol, f"bfloat16 {what}"
        row_err = (got_b.double().cpu() - wide).abs().amax(-1) / wide.abs().max()
        assert float(row_err.mean()) <= 6e-2 and float(row_err.median()) <= 3e-2, f"bfloat16 {what}: rows in the mean"


def window_edges(env, name, window_layer, at=90):
    """A query just inside and just outside a window: the token whose key lies exactly at the edge is changed, in a prompt and with
    the query decoded alone. In a model of that one layer, run once, the logits move inside the window and stay outside. Of all
    tokens that may stand at the edge, the pair whose keys matter most to the query at the edge is taken."""
    window = CONFIGS[name]["layers"][window_layer]["mixer"]["mask"]["size"]
    V = CONFIGS[name]["vocab"]
    ids = random_ids(at + window + 2, V, 640)
    folder, edge = env.folders(name), at + window - 1
    rows = []
    for token in range(V):
        ids[at] = token
        rows.append(plain_logits(folder, ids[:edge + 1])[edge])
    apart = (torch.stack(rows)[:, None] - torch.stack(rows)[None]).abs().amax(-1)
    one, two = divmod(int(apart.argmax()), V)
    other = list(ids)
    ids[at], other[at] = one, two
    shows = float(apart.max() / torch.stack(rows).abs().max())
    assert shows > 1e-2, "no key at the edge matters"
    out = {}
    for key, tokens in (("a", ids), ("b", other)):
        runner, manager, folder = env.runner(name, 2 * -(-len(ids) // PAGE[name]), 2)
        d = Driver(runner, manager)
        d.step({"w": tokens})
        cut = at + window - 2
        d.step({"r": tokens[:cut]})
        for t in range(cut, len(tokens)):
            d.step({"r": tokens[t:t + 1]})
        out[key] = (d.result("w"), d.result("r"))
        for got in out[key]:
            CUTS.check(env, folder, tokens, got, f"{name} window edge")
    for a, b in zip(out["a"], out["b"]):
        moved = (a - b).abs().amax(-1) / a.abs().max()
        assert float(moved[edge]) > 0.3 * shows, "the last query that sees the key"
        assert float(moved[edge + 1]) == 0, "the first query that does not"
