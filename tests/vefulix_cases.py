"""Test configurations of the Vefulix design, all the tests' own, and their plain evaluation (tests/plain_vefulix.py).

The configurations differ from each other in every size: the three mixers in several orders, one to seven residual streams,
layers without a feed-forward, experts with and without a shared one, one expert per token and all of them, sizes that are
no whole steps of 8, single heads, one tap, heads that share keys and heads that do not. `make_folder` draws weights whose
rows have unit size on unit inputs, so that sublayers matter beside the streams, score scales are large, so that the softmax
is peaked and a key that is wrongly seen or missed moves the logits, and biases, sinks and routers are scaled up so that
leaving one out moves them far beyond the tolerance.
"""
from __future__ import annotations

import os

import torch

import helpers
import plain_vefulix
from cut_cases import Cuts
from helpers import Driver, random_ids, rel_err
from mini_engine_amd.config.model_config import VefulixConfig
from mini_engine_amd.weights.random_init import write_random_model


def _mlstm(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def _latent(heads, dim, vdim, q_rank, kv_rank, scale):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}}


def _moe(ff, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
    return mlp


def _with(layer, mlp):
    return dict(layer, mlp=mlp)


def _model(vocab, width, eps, streams, layers, cap=None):
    d = {"architecture": "Vefulix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams, "layers": layers}
    if cap is not None:
        d["logit_softcap"] = cap
    return d


def _real(moe):
    return [_with(_delta(8, 4, 128, 128, 4), moe), _with(_latent(16, 128, 128, 384, 256, 128 ** -0.5 * 2), moe),
            _with(_mlstm(4, 128, 256, 15.0), moe), _with(_latent(16, 128, 64, 320, 128, 128 ** -0.5), moe)]


CONFIGS = {
    "mix": _model(101, 48, 1e-5, 2, [
        _with(_delta(4, 2, 8, 16, 3), _moe(24, 8, 3, 40)),
        _with(_latent(3, 16, 24, 24, 40, 0.8), _moe(16, 6, 2)),
        _with(_mlstm(3, 8, 16, 5.0), _moe(24, 8, 3, 32)),
        _with(_latent(2, 24, 16, 32, 24, 0.7), None),
    ], 12.0),
    # sizes in no whole steps of 8; a layer without a feed-forward first; every expert chosen; a softcap that hardly bends
    "odd": _model(97, 36, 1e-6, 5, [
        _with(_mlstm(3, 10, 14, 3.0), None),
        _with(_delta(6, 2, 10, 6, 5), _moe(20, 6, 1)),
        _with(_latent(3, 12, 10, 18, 20, 1.0), _moe(12, 5, 5, 20)),
        _with(_delta(3, 3, 6, 18, 2), _moe(9, 3, 2, 11)),
        _with(_mlstm(2, 14, 9, 8.0), _moe(10, 7, 4)),
    ], 90.0),
    # what a model may make equal or one: one stream, one head, one tap, one expert per token, no cap on the logits
    "one": _model(64, 32, 1e-5, 1, [
        _with(_delta(1, 1, 16, 16, 1), _moe(16, 4, 1)),
        _with(_latent(1, 16, 16, 16, 16, 1.2), _moe(16, 1, 1, 16)),
        _with(_mlstm(1, 16, 16, 2.0), _moe(16, 2, 1)),
        _with(_delta(2, 2, 8, 8, 4), None),
    ]),
    # a width in whole 16-byte pieces around sizes that are not (the kernels' vector paths beside their scalar ones in one
    # model); a number of streams without a kernel of its own; two latent layers of different ranks
    "mid": _model(120, 64, 1e-5, 7, [
        _with(_latent(5, 10, 14, 27, 22, 0.9), _moe(24, 2, 2, 16)),
        _with(_mlstm(4, 20, 24, 6.0), _moe(12, 9, 4, 28)),
        _with(_latent(1, 16, 24, 40, 48, 0.8), None),
        _with(_delta(6, 3, 12, 20, 7), _moe(16, 4, 2)),
    ], 20.0),
    # no latent layer: a model without any pages
    "flat": _model(50, 24, 1e-5, 3, [
        _with(_mlstm(2, 4, 6, 4.0), _moe(16, 4, 2)),
        _with(_delta(2, 1, 12, 8, 3), None),
    ], 15.0),
    # no recurrence: a model without any state
    "pages": _model(70, 40, 1e-5, 2, [
        _with(_latent(2, 16, 8, 24, 32, 1.1), _moe(16, 4, 2)),
        _with(_latent(4, 8, 16, 16, 24, 1.4), _moe(24, 3, 1, 16)),
    ], 25.0),
    # the layer sizes of a real model (GPU only); every token takes all 4 experts, so that no choice can fall otherwise in bfloat16
    # than in float32 and every row can be held to the tolerance
    "real": _model(2048, 1024, 1e-6, 4, _real(_moe(384, 4, 4, 1536)), 30.0),
    # the same with 4 of 32 experts per token: a token whose choice hangs on two close logits may choose otherwise in bfloat16,
    # so these rows are held to the tolerance in the mean
    "routed": _model(2048, 1024, 1e-6, 4, _real(_moe(384, 32, 4, 1536)), 30.0),
}
SEEDS = {"mix": 41, "odd": 42, "one": 43, "mid": 44, "flat": 45, "pages": 46, "real": 47, "routed": 48}
PAGE = {"mix": 16, "odd": 8, "one": 4, "mid": 32, "flat": 16, "pages": 16, "real": 16, "routed": 16}
SMALL = ("mix", "odd", "one", "mid", "flat", "pages")


def _every_expert(config):
    """The configuration with every expert chosen by every token: no choice can then fall otherwise in bfloat16 than in float32."""
    layers = [l if l["mlp"] is None else dict(l, mlp=dict(l["mlp"], router=dict(l["mlp"]["router"], top=l["mlp"]["router"]["experts"])))
              for l in config["layers"]]
    return dict(config, layers=layers)


for _name in SMALL:
    CONFIGS[_name + "-all"], SEEDS[_name + "-all"], PAGE[_name + "-all"] = _every_expert(CONFIGS[_name]), SEEDS[_name], PAGE[_name]


def make_folder(name: str, path: str) -> str:
    """A checkpoint of the configuration with seeded random weights in bfloat16, reshaped so that every mechanism shows (see
    the module's text)."""
    from safetensors import safe_open
    from safetensors.torch import save_file

    cfg = VefulixConfig.from_dict(CONFIGS[name])
    write_random_model(cfg, SEEDS[name], path, torch.bfloat16)
    file = os.path.join(path, "model.safetensors")
    with safe_open(file, "pt", device="cpu") as f:
        tensors = {k: f.get_tensor(k) for k in f.keys()}
    for k in tensors:
        t = tensors[k].float()
        last = k.rsplit(".", 1)[1] if "." in k else k
        if k.endswith(".sink"):
            t = 1.0 + 2.0 * torch.arange(t.numel(), dtype=torch.float32) / max(1, t.numel() - 1) if t.numel() > 1 else t + 2.0
        elif ".hc" in k:
            g = torch.Generator().manual_seed(sum(map(ord, k)))        # shares far from even, from and to not alike
            t = t + 0.4 * (torch.rand(t.shape, generator=g) - 0.5)
        elif k.endswith(".router.b") or k.endswith(".i.b"):
            t = t * 50.0
        elif k.endswith(".f.b"):
            t = t - 3.0                                                # forget gates that forget within a few tokens to a few dozen
        elif k.endswith("norm.b") or k.endswith("norm1.b") or k.endswith("norm2.b"):
            t = t * 3.0
        elif k.endswith(".conv"):
            t = t * 2.0
        elif k == "embed":
            t = t * 50.0
        elif t.dim() == 2:
            t = t / (0.02 * t.shape[1] ** 0.5)                         # unit outputs on unit inputs
            if last == "router":
                t = t * 2.0
            elif k == "head":
                t = t * 4.0
        tensors[k] = t.to(tensors[k].dtype)
    save_file(tensors, file, metadata={"format": "pt"})
    return path


_plain: dict = {}


def plain_model(folder: str):
    if folder not in _plain:
        _plain[folder] = plain_vefulix.read_folder(folder)
    return _plain[folder]


def plain_logits(folder: str, ids: list) -> torch.Tensor:
    key = (folder, tuple(ids))
    if key not in _plain:
        cfg, w = plain_model(folder)
        _plain[key] = plain_vefulix.logits(cfg, w, ids)
    return _plain[key]


CUTS = Cuts(CONFIGS, PAGE, plain_logits)


def layers_one_by_one(env, name):
    """The sum of the streams after every layer, float32, against the plain evaluation's."""
    runner, manager, folder = env.runner(name, -(-19 // PAGE[name]), 1)
    ids = random_ids(19, CONFIGS[name]["vocab"], 77)
    cfg, w = plain_model(folder)
    _, want = plain_vefulix.forward(cfg, w, ids, keep_layers=True)
    got, inner = [], runner.model.layers
    kept = [layer.forward for layer in inner]

    def spy(forward):
        def run(*a):
            h, streams = forward(*a)
            got.append(h.settle(streams))
            return h, streams
        return run

    try:
        for layer in inner:
            layer.forward = spy(layer.forward)
        Driver(runner, manager).step({"r": ids}, end=["r"])
    finally:
        for layer, forward in zip(inner, kept):
            layer.forward = forward
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert a.dtype == torch.float32 and rel_err(a, b) <= env.tol, f"{name}: layer {i} ({cfg['layers'][i]['type']}): {rel_err(a, b):.3g}"


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
