"""Venezen on the CPU: configuration, checkpoint layout, the run order with its loop, and the engine's bookkeeping for it (pages of
a latent beside windows, pages per pass, batches, cuts, the scheduler) with the plain twins of the kernels in float32, against the
plain evaluation; each new twin against the plain function of its mechanism; and the plain evaluation with one mechanism taken
out, which must be far off (so that the random weights cannot hide a fault of that mechanism)."""
import copy
import json

import pytest
import torch

import kernel_twins as twin
import plain_venezen as P
import venezen_cases as C
from mini_engine_amd.cache.manager import CacheManager
from mini_engine_amd.config.model_config import ConfigError, VenezenConfig, load_model_config
from mini_engine_amd.engine.runner import ModelRunner
from mini_engine_amd.kernels import ops
from mini_engine_amd.parts.base import Biased, ScaledSum, Settled, TermSum, make_part
from mini_engine_amd.parts.block import with_start
from mini_engine_amd.registry import build_model
from mini_engine_amd.weights.loader import WeightError, load_model

CUTS = C.CUTS


@pytest.fixture(scope="module")
def venezen_folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = C.make_folder(name, str(tmp_path_factory.mktemp(f"venezen_{name}")))
        return made[name]

    return get


class Env:
    device, dtype, tol = "cpu", torch.float32, 4e-5      # float32 sums against float64

    def __init__(self, folders):
        self.folders, self.models = folders, {}

    def runner(self, name, pages, slots):
        folder = self.folders(name)
        if name not in self.models:
            self.models[name] = load_model(folder, self.device, self.dtype, 512)
        model = self.models[name]
        manager = CacheManager(pages, C.PAGE[name], ModelRunner.windows_of(model), num_state_slots=0, enable_prefix_caching=False)
        return ModelRunner(model, manager, self.dtype, self.device, 512, poison_cache=True), manager, folder


def test_config_reads_back_and_refuses_what_it_cannot_run(tmp_path):
    for name, raw in C.CONFIGS.items():
        cfg = VenezenConfig.from_dict(raw)
        assert VenezenConfig.from_dict(cfg.to_dict()) == cfg
        assert len(cfg.layers) == len(raw["layers"]) and cfg.vocab_size == raw["vocab"]
        assert cfg.run_order() == P.run_order(raw)
    with open(tmp_path / "config.json", "w") as f:
        json.dump(C.CONFIGS["mix"], f)
    assert isinstance(load_model_config(str(tmp_path)), VenezenConfig)          # chosen by the file's architecture name
    alone = copy.deepcopy(C.CONFIGS["mix"])
    alone["layers"][1]["mixer"].pop("kv_heads")
    alone["layers"][1]["mlp"]["router"].pop("identity")
    got = VenezenConfig.from_dict(alone).layers[1]
    assert got.mixer["kv_heads"] == 4 and got.mlp["identity"] == 0              # absent: a key of its own per head, no identity experts
    for spoil in (lambda c: c["layers"][0].update(type="latent"),
                  lambda c: c["layers"][0]["mixer"].update(rot_dim=7),
                  lambda c: c["layers"][0]["mixer"]["rot"].update(dims=4),
                  lambda c: c["layers"][0]["mixer"].pop("rot"),
                  lambda c: c["layers"][0]["mixer"].pop("kv_rank"),
                  lambda c: c["layers"][1]["mixer"].update(kv_heads=3),
                  lambda c: c["layers"][1]["mixer"].update(vdim=8),
                  lambda c: c["layers"][1]["mixer"]["mask"].update(size=0),
                  lambda c: c["layers"][1]["mixer"].update(scale=0.0),
                  lambda c: c["layers"][1]["mlp"]["router"].update(top=9),
                  lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"),
                  lambda c: c["layers"][1]["mlp"]["shared"].update(limit=0.0),
                  lambda c: c["layers"][1]["mlp"].update(kind="sparse"),
                  lambda c: c["loop"].update(stop=5),
                  lambda c: c["loop"].update(times=0),
                  lambda c: c["norm"].pop("eps")):
        bad = copy.deepcopy(C.CONFIGS["mix"])
        spoil(bad)
        with pytest.raises(ConfigError):
            VenezenConfig.from_dict(bad)


def test_model_is_assembled_from_the_config(venezen_folders, tmp_path):
    model = build_model(VenezenConfig.from_dict(C.CONFIGS["mix"]))
    assert [(c.layer, c.add_start) for c in model.order] == [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    plan = model.cache_plan()
    assert all(plan.call_writes) and len(plan.call_group) == 6                   # each pass has pages of its own
    assert plan.call_group[1] == plan.call_group[3] and plan.call_index_in_group[1] != plan.call_index_in_group[3]
    assert plan.group_needs[plan.call_group[1]].keep() == 21 and plan.group_needs[plan.call_group[0]].keep() is None
    assert plan.group_needs[plan.call_group[0]].tensors[0].shape[2] == 48       # a rank of 40 with 8 rotating
    assert model.layers[1].mixer.qkv.out_features == (4 + 2) * 16                # no value projection
    assert model.layers[2].feed_forward.shared is None and model.layers[3].feed_forward is None
    assert model.layers[1].feed_forward.router is None and dict((n, s.shape) for n, _, _, s in model.layers[1].named_specs())["feed_forward.router"] == (8, 48)
    assert model.head.tied_to is model.embedding
    names = {src.name for sources in model.weight_sources.values() for src in sources}
    assert {"embed", "final.norm", "l0.mix.q", "l0.mix.dkv", "l0.mix.dkv.norm", "l0.mix.uk", "l0.mix.uv", "l0.mix.o", "l0.mlp.gate.b", "l0.mlp.down.b",
            "l1.mix.k", "l1.mlp.e5.gate", "l1.mlp.router", "l1.mlp.correction", "l1.mlp.shared.down", "l3.norm1"} <= names
    assert not {"l1.mix.v", "head", "l1.mlp.e6.gate", "l2.mlp.shared.up", "l3.norm2", "l0.norm1.b"} & names
    # a checkpoint of another shape is refused as a whole
    from safetensors.torch import load_file, save_file
    tensors = load_file(venezen_folders("mix") + "/model.safetensors")
    tensors["l0.mix.uk"] = tensors["l0.mix.uk"][:-1].contiguous()
    tensors["l9.extra"] = tensors.pop("l1.mlp.correction")
    save_file(tensors, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(C.CONFIGS["mix"]))
    with pytest.raises(WeightError) as e:
        load_model(str(tmp_path), "cpu", torch.float32, 64)
    assert all(n in str(e.value) for n in ("l0.mix.uk", "l9.extra", "l1.mlp.correction"))


def test_parts_refuse_what_does_not_fit_together():
    attention = lambda **kw: make_part("mixer", "attention", hidden_size=16, num_heads=2, num_kv_heads=2, head_dim=8, scale=1.0, **kw)
    for bad in (dict(values_are_keys=True, own_kv=False), dict(values_are_keys=True, value_dim=4), dict(values_are_keys=True, qkv_bias=True),
                dict(sinks=True, sink_score=0.0), dict(slopes=[0.5]), dict(slopes=[0.5, -0.1]), dict(slopes=[0.5, 0.1], qkv_bias=True)):
        with pytest.raises(ValueError):
            attention(**bad)
    moe = lambda **kw: make_part("feed_forward", "moe", hidden_size=16, intermediate_size=8, num_experts=4, top=2, **kw)
    for bad in (dict(identity=-1), dict(clamp=(0.0, 1.0)), dict(gated=False, clamp=(1.0, 1.0)), dict(identity=1, group_count=2, group_keep=1)):
        with pytest.raises(ValueError):
            moe(**bad)


# ---------------------------------------------------------------- each twin against the plain function of its mechanism

def _paged(T, page, *shapes):
    n = -(-T // page)
    return [torch.full((n + 1,) + s, float("nan")) for s in shapes], torch.arange(n, dtype=torch.int32)[None]


def test_attention_twins_whose_values_are_keys_against_the_plain_heads():
    """Slopes, a sink that scores 0, a window; the key at the window's edge stands out for one query, so that an edge that is one
    off shows."""
    torch.manual_seed(1)
    T, H, G, D, width, page, window = 30, 6, 2, 8, 12, 4, 9
    m = {"heads": H, "kv_heads": G, "dim": D, "scale": 0.7, "mask": {"size": window}}
    h = torch.randn(T, width, dtype=torch.float64)
    w = {"x.q": torch.randn(H * D, width).double(), "x.k": torch.randn(G * D, width).double(), "x.o": torch.eye(H * D).double()}
    k = h[20] @ w["x.k"].T
    for at in (28, 29):                      # head 5 of the queries at 28 (sees 20) and 29 (does not) asks for the key of position 20
        w["x.q"][5 * D:] += 0.5 * torch.outer(k[D:], h[at]) / (h[at] @ h[at])
    want = P.attention(h, w, "x.", m, 1e-5)
    rows = torch.cat((h @ w["x.q"].T, h @ w["x.k"].T), 1).float()
    (kc, vc), bt = _paged(T, page, (G, page, D), (G, D, page))
    pos = torch.arange(T, dtype=torch.int32)
    twin.qk_norm_rope_store(rows, None, None, 0.0, None, pos, pos, kc, vc, H, G, D, page, values_are_keys=True)
    slopes, sinks = torch.tensor(P.slopes(H), dtype=torch.float32), torch.zeros(H)
    run = lambda win: twin.paged_attention(rows[:, :H * D], kc, vc, page, bt, torch.tensor([T], dtype=torch.int32), torch.zeros(T, dtype=torch.int32), pos,
                                           torch.tensor([0, T], dtype=torch.int32), 0, 0, 0.7, win, H, G, D, sinks=sinks, slopes=slopes)
    assert float((run(window).double() - want).abs().max()) < 2e-5 * float(want.abs().max())
    for off, at in ((window - 1, 28), (window + 1, 29)):
        assert float((run(off)[at].double() - want[at]).abs().max()) > 1e-1 * float(want.abs().max())
    # one decoded token at a time through the fused step's twin
    (kc, vc), bt = _paged(T, page, (G, page, D), (G, D, page))
    fresh = torch.cat((h @ w["x.q"].T, h @ w["x.k"].T), 1).float()
    got = torch.cat([twin.decode_step_attention(fresh[t:t + 1], None, None, 0.0, None, kc, vc, page, bt, torch.tensor([t + 1], dtype=torch.int32), t + 1,
                                                0.7, window, H, G, D, sinks=sinks, slopes=slopes, values_are_keys=True) for t in range(T)])
    assert float((got.double() - want).abs().max()) < 2e-5 * float(want.abs().max())


def test_values_are_the_keys_in_front_of_norm_and_rotation(plain_backend):
    """Another design may norm and rotate such keys: the values stay as projected."""
    torch.manual_seed(2)
    T, H, G, D, page = 5, 2, 1, 8, 4
    rows = torch.randn(T, (H + G) * D)
    raw = rows[:, H * D:].clone()
    (kc, vc), _ = _paged(T, page, (G, page, D), (G, D, page))
    table = make_part("position_encoding", "rotary", head_dim=D, theta=100.0)
    table.finalize("cpu", torch.float32, 16)
    pos = torch.arange(T, dtype=torch.int32)
    twin.qk_norm_rope_store(rows, torch.ones(D), torch.ones(D), 1e-5, table.table, pos, pos, kc, vc, H, G, D, page, values_are_keys=True)
    assert torch.equal(vc.permute(0, 3, 1, 2).reshape(-1, D)[:T], raw) and not torch.allclose(kc.transpose(1, 2).reshape(-1, D)[:T], raw)


@pytest.mark.parametrize("query_rank", [None, 6])
def test_latent_rows_of_half_split_pairs_become_adjacent_once(plain_backend, query_rank):
    """The rotating rows are moved when the weights are bound, once, in the queries' projection and the shared key's: the scores of
    rotated parts are those of the pairs as stored."""
    torch.manual_seed(3)
    H, dn, dr, R, width, T = 2, 4, 6, 5, 7, 9
    enc = make_part("position_encoding", "rotary", head_dim=dr, theta=50.0, exact_angles=True)
    part = make_part("mixer", "latent_attention", hidden_size=width, num_heads=H, nope_dim=dn, rot_dim=dr, value_dim=3, rank=R, scale=1.0,
                     norm_eps=1e-5, position=enc, query_rank=query_rank)
    for _, owner, local, spec in part.named_specs():
        owner.set_param(local, torch.randn(spec.shape))
    q_rows = (part.uq if query_rank else part.in_proj).weight[:H * (dn + dr)].clone()
    kv_rows = part.in_proj.weight[part.kv_at:part.kv_at + R + dr].clone()
    for p in part.parts():
        p.finalize("cpu", torch.float32, T)
    once = part.in_proj.weight.clone()
    part.finalize("cpu", torch.float32, T)                       # a second time changes nothing
    assert torch.equal(part.in_proj.weight, once)
    x, xq, pos = torch.randn(T, width).double(), torch.randn(T, query_rank or width).double(), torch.arange(T)
    want_q = P.rotate_halves((xq @ q_rows.double().T).view(T, H, dn + dr)[..., dn:], pos, 50.0)
    want_k = P.rotate_halves((x @ kv_rows.double().T)[:, None, R:], pos, 50.0)[:, 0]
    D = part.head_dim
    kc, vc = torch.zeros(3, 1, 4, D), torch.zeros(3, 1, D, 4)
    q_now = xq.float() @ (part.uq if query_rank else part.in_proj).weight[:H * (dn + dr)].T
    rows = torch.cat((q_now, x.float() @ part.in_proj.weight[part.kv_at:part.kv_at + R + dr].T), 1)
    qa = twin.latent_prepare(rows, 0, H * (dn + dr), H, dn, dr, R, D, torch.ones(R), 1e-5, enc.table, pos.int(), pos.int(), kc, vc, 4)
    got_q = qa.view(T, H, D)[:, :, R:R + dr].double()
    got_k = kc.view(-1, D)[:T, R:R + dr].double()
    assert torch.allclose(torch.einsum("thd,sd->hts", got_q, got_k), torch.einsum("thd,sd->hts", want_q, want_k), atol=1e-4)
    assert torch.equal(q_now.view(T, H, dn + dr)[..., :dn], (xq.float() @ q_rows.T).view(T, H, dn + dr)[..., :dn])


def test_expert_twins_with_identity_experts_and_a_clamped_gate_against_the_plain_mixture():
    torch.manual_seed(4)
    T, n, F, E, Z = 40, 10, 6, 4, 3
    h = torch.randn(T, n).double()
    w = {"x.router": torch.randn(E + Z, n).double(), "x.correction": torch.randn(E + Z).double() * 0.3}
    for e in range(E):
        w |= {f"x.e{e}.gate": torch.randn(F, n).double(), f"x.e{e}.up": torch.randn(F, n).double(), f"x.e{e}.down": torch.randn(n, F).double()}
    gate_up = torch.stack([torch.cat((w[f"x.e{e}.gate"], w[f"x.e{e}.up"])) for e in range(E)]).float()
    down = torch.stack([w[f"x.e{e}.down"] for e in range(E)]).float()
    for top in (1, 3, E + Z):
        f = {"router": {"experts": E, "top": top, "identity": Z, "scale": 1.7}, "expert": {"limit": 0.8}}
        want = P.mixture(h, w, "x.", f)
        rule = ops.RouteRule("softmax", correction=w["x.correction"].float(), normalise=True, scale=1.7)
        got = twin.route_and_run_experts(h.float(), w["x.router"].float(), top, 1, 1, gate_up, down, rule=rule, clamp=(0.8, 1.702))
        assert got.shape == (top, T, n) and torch.allclose(got.sum(0).double(), want, atol=1e-4)
        ids, _ = twin.moe_route(h.float(), w["x.router"].float(), top, 1, 1, rule)
        assert (ids >= E).any() and (ids < E).any()


def test_dense_part_with_biases(plain_backend):
    torch.manual_seed(5)
    T, n, F = 7, 10, 12
    w = {f"x.{k}": torch.randn(*s).double() for k, s in (("gate", (F, n)), ("up", (F, n)), ("down", (n, F)), ("gate.b", (F,)), ("up.b", (F,)), ("down.b", (n,)))}
    part = make_part("feed_forward", "swiglu", hidden_size=n, intermediate_size=F, bias=True)
    part.gate_up.set_param("weight", torch.cat((w["x.gate"], w["x.up"])).float())
    part.down.set_param("weight", w["x.down"].float())
    part.set_param("gate_up_bias", torch.cat((w["x.gate.b"], w["x.up.b"])).float())
    part.set_param("down_bias", w["x.down.b"].float())
    h = torch.randn(T, n).double()
    want = P.dense(h, w, "x.")
    assert torch.allclose(part.forward(h.float()).double(), want, atol=1e-5)
    part.defer_bias = True
    got = part.forward(h.float())
    assert isinstance(got, Biased) and torch.allclose((got.rows + got.bias).double(), want, atol=1e-5)


def test_sums_that_wait_for_the_next_norm(plain_backend):
    """Terms, partial sums and biases, in one pass or (more than four) several, in front of either norm, of another kind of block, of
    the final norm at chosen rows, and with the embedding's output added once more."""
    torch.manual_seed(6)
    T, n = 5, 12
    stream = torch.randn(T, n)
    terms = [torch.randn(T, n), torch.randn(3, T, n), Biased(torch.randn(2, T, n), torch.randn(n)), torch.randn(T, n), torch.randn(T, n), torch.randn(T, n)]
    total = stream + sum((t.rows.sum(0) + t.bias) if isinstance(t, Biased) else (t.sum(0) if t.dim() == 3 else t) for t in terms)
    layer, rms = make_part("norm", "layer", size=n, eps=1e-4, bias=False), make_part("norm", "rms", size=n, eps=1e-4)
    for norm in (layer, rms):
        norm.set_param("weight", torch.rand(n) + 0.5)
        norm.finalize("cpu", torch.float32, 8)
    want = {layer: P.layer_norm(total.double(), layer.weight.double(), 1e-4), rms: P.unit_rms(total.double(), 1e-4) * rms.weight.double()}
    for norm in (layer, rms):
        y, new = TermSum(terms).normed(norm, stream)
        assert torch.allclose(y.double(), want[norm], atol=1e-5) and torch.allclose(new, total, atol=1e-5)
        rows = torch.tensor([3, 0], dtype=torch.int32)
        assert torch.allclose(TermSum(terms).normed_rows(stream, norm, rows).double(), want[norm][[3, 0]], atol=1e-5)
    assert torch.allclose(TermSum(terms).settle(stream), total, atol=1e-5)
    start = torch.randn(T, n)
    for left, residual, base in ((TermSum(terms), stream, total), (terms[0], stream, stream + terms[0]), (terms[1], stream, stream + terms[1].sum(0)),
                                 (Settled(None), stream, stream), (ScaledSum([(terms[0], None)], 0.5), stream, stream + 0.5 * terms[0])):
        h, r = with_start(left, residual, start)
        assert torch.allclose(h.settle(r), base + start, atol=1e-5)
    # a block of another kind takes the settled stream
    class Double(torch.nn.Module):
        def forward(self, x, *a):
            return 2.0 * x
    for kind, norms in (("output_norm", dict(norm1=rms)), ("parallel", dict(norm1=rms)), ("hyper_connected", dict(norm1=rms, streams=1))):
        block = make_part("block", kind, mixer=make_part("mixer", "mlstm", hidden_size=n, num_heads=1, key_dim=4, value_dim=4, gate_cap=4.0, norm_eps=1e-5), **norms)
        block.mixer = Double()
        if kind == "hyper_connected":
            block.read1, block.out1, block.mix1 = torch.ones(1), torch.ones(1), torch.ones(1, 1)
        from mini_engine_amd.parts.block import settled
        h, r = settled(*block.forward(TermSum(terms), stream, None, None, None))
        inner = (total + rms.weight * P.unit_rms(2.0 * total, 1e-4)) if kind == "output_norm" else total + 2.0 * want[rms].float()
        assert torch.allclose(r, inner.float(), atol=1e-4), kind


# ---------------------------------------------------------------- a mechanism left out must show

def _zero(name):
    return lambda cfg, w: w.update({name: torch.zeros_like(w[name])})


def _mixer(i, **kw):
    return lambda cfg, w: cfg["layers"][i]["mixer"].update(kw)


SPOILS = {
    "embedding_scale": lambda cfg, w: cfg["embedding"].update(scale=1.0), "passes": lambda cfg, w: cfg["loop"].update(times=1),
    "loop_start": lambda cfg, w: cfg["loop"].update(start=0), "loop_stop": lambda cfg, w: cfg["loop"].update(stop=4),
    "latent_norm": lambda cfg, w: w.update({"l0.mix.dkv.norm": torch.ones_like(w["l0.mix.dkv.norm"])}),
    "rotation_base": lambda cfg, w: cfg["layers"][2]["mixer"]["rot"].update(base=1000.0), "latent_scale": _mixer(0, scale=0.5),
    "shared_key_part": lambda cfg, w: w.update({"l0.mix.dkv": torch.cat((w["l0.mix.dkv"][:40], torch.zeros_like(w["l0.mix.dkv"][40:])))}),
    "norm1": lambda cfg, w: w.update({"l1.norm1": torch.ones_like(w["l1.norm1"])}), "final_norm": lambda cfg, w: w.update({"final.norm": torch.ones_like(w["final.norm"])}),
    "score_scale": _mixer(1, scale=0.6), "window_longer": _mixer(1, mask={"size": 22}), "window_shorter": _mixer(1, mask={"size": 20}),
    "shared_keys": lambda cfg, w: w.update({"l1.mix.k": w["l1.mix.k"].roll(16, 0)}),
    "gate_bias": _zero("l0.mlp.gate.b"), "up_bias": _zero("l0.mlp.up.b"), "down_bias": _zero("l0.mlp.down.b"),
    "correction": _zero("l1.mlp.correction"), "router_scale": lambda cfg, w: cfg["layers"][1]["mlp"]["router"].update(scale=1.0),
    "top": lambda cfg, w: cfg["layers"][1]["mlp"]["router"].update(top=2), "limit": lambda cfg, w: cfg["layers"][1]["mlp"]["expert"].update(limit=9.0),
    "shared_limit": lambda cfg, w: cfg["layers"][1]["mlp"]["shared"].update(limit=9.0), "shared_expert": lambda cfg, w: cfg["layers"][1]["mlp"].pop("shared"),
    "expert_weights": _zero("l2.mlp.e0.down"),
}
SWAPS = {
    "start_again": ("run_order", lambda real: lambda cfg: [(i, False) for i, _ in real(cfg)]),
    "pairs": ("rotate_halves", lambda real: lambda x, pos, base: real(torch.cat((x[..., 0::2], x[..., 1::2]), -1), pos, base)),
    "no_rotation": ("rotate_halves", lambda real: lambda x, pos, base: x),
    "mean": ("layer_norm", lambda real: lambda x, w, eps: P.unit_rms(x, eps) * w),
    "no_slopes": ("slopes", lambda real: lambda H: [0.0] * H), "slopes_turned": ("slopes", lambda real: lambda H: real(H)[::-1]),
    "slope_step": ("slopes", lambda real: lambda H: [2.0 ** (-8.0 * a / H) for a in range(H)]),
    "no_sink": ("softmax_plus_one", lambda real: lambda s: torch.softmax(s, -1)),
    "weights_with_correction": ("choose", lambda real: lambda s, c, top, scale: real(s + c, 0 * c, top, scale)),
    "not_normalised": ("choose", lambda real: lambda s, c, top, scale: (real(s, c, top, 1.0)[0], s.gather(-1, real(s, c, top, 1.0)[0]) * scale)),
    "identity_silent": ("mixture", lambda real: lambda h, w, pre, f: real(h, w, pre, f) - real(h, dict(w, **{k: torch.zeros_like(v) for k, v in w.items() if k.startswith(pre) and k.endswith(".down")}), pre, f)),
    "gate_without_one": ("clamped_expert", lambda real: lambda h, w, pre, limit: real(h, w, pre, limit) - real(h, dict(w, **{pre + "up": torch.zeros_like(w[pre + "up"])}), pre, limit)),
}


@pytest.mark.parametrize("spoil", [*SPOILS, *SWAPS])
def test_the_weights_show_a_mechanism_that_is_left_out(venezen_folders, monkeypatch, spoil):
    cfg, w = P.read_folder(venezen_folders("mix"))
    ids = C.random_ids(40, 103, 5)
    ref = P.logits(cfg, w, ids)
    cfg, w = copy.deepcopy(cfg), dict(w)
    if spoil in SPOILS:
        SPOILS[spoil](cfg, w)
    else:
        name, swap = SWAPS[spoil]
        real = getattr(P, name)
        monkeypatch.setattr(P, name, swap(real))
        if name in P.MIXERS:
            monkeypatch.setitem(P.MIXERS, name, getattr(P, name))
    moved = float((P.logits(cfg, w, ids) - ref).abs().max() / ref.abs().max())
    assert moved > 3e-3, f"leaving out {spoil} hardly shows in the logits: {moved:.2g}"


def test_keys_far_away_show_in_the_logits(venezen_folders):
    """In the model of latent layers alone, an early token that some later query asks for moves that query's logits hundreds of
    positions on; so a lost page or key cannot hide."""
    cfg, w = P.read_folder(venezen_folders("pages"))
    ids = C.random_ids(330, 70, 600)
    ref = P.logits(cfg, w, ids)
    moved = torch.zeros(330)
    for at in (0, 15, 16, 40):
        other = list(ids)
        other[at] = (other[at] + 1) % 70
        moved = torch.maximum(moved, ((P.logits(cfg, w, other) - ref).abs().amax(-1) / ref.abs().max()).float())
    assert float((moved[200:] > 1e-3).float().mean()) > 0.5


# ---------------------------------------------------------------- the engine against the plain evaluation

@pytest.mark.parametrize("name", C.SMALL)
def test_every_layer(venezen_folders, plain_backend, name):
    C.layers_one_by_one(Env(venezen_folders), name)


@pytest.mark.parametrize("name", C.SMALL)
@pytest.mark.parametrize("case", CUTS.ALL, ids=lambda c: c.__name__)
def test_cuts(venezen_folders, plain_backend, case, name):
    case(Env(venezen_folders), name)


@pytest.mark.parametrize("name", ["pages", "mix"])
def test_long_prompts(venezen_folders, plain_backend, name):
    CUTS.long_prompt(Env(venezen_folders), name)


@pytest.mark.parametrize("size", [1, 2, 7, 8, 9, 40])
def test_window_edges(tmp_path_factory, plain_backend, size):
    C.window_edges(Env(edge_folder(tmp_path_factory, size)), f"edge{size}", 0)


def edge_folder(tmp_path_factory, size):
    """A model of one windowed layer: what lies outside its window cannot reach a logit by any other way."""
    name = f"edge{size}"
    C.CONFIGS[name] = C._model(40, 16, 1e-5, 2.0, [C._with(C._attention(3, 1, 16, size, 1.0), None)])
    C.SEEDS[name], C.PAGE[name] = 60 + size, 8
    path = C.make_folder(name, str(tmp_path_factory.mktemp(name)))
    return lambda _: path


@pytest.mark.parametrize("name", ["mix", "odd", "windows"])
def test_greedy_generation_through_the_scheduler(venezen_folders, plain_backend, name):
    CUTS.greedy_through_the_engine("cpu", "float32", name, venezen_folders(name), exact=True)


def test_command_line_on_a_folder_of_this_design(venezen_folders, plain_backend, tmp_path):
    """`python -m mini_engine_amd.cli --model DIR`: the folder's config picks the model class; prompts in, greedy tokens out."""
    from mini_engine_amd import cli
    folder = venezen_folders("mix")
    prompts = [C.random_ids(n, 103, 950 + n) for n in (3, 19, 41)]
    path = tmp_path / "prompts.jsonl"
    path.write_text("\n".join(json.dumps(p) for p in prompts) + "\n")
    out = tmp_path / "tokens.jsonl"
    rc = cli.main(["--model", folder, "--prompts", str(path), "--tokens-out", str(out), "--temperature", "0", "--max-output", "6",
                   "--dtype", "float32", "--device", "cpu", "--num-kv-blocks", "64", "--block-size", "8", "--budget", "16",
                   "--max-num-seqs", "2", "--max-model-len", "128", "--out", str(tmp_path / "rows.jsonl")])
    assert rc == 0
    got = [json.loads(line) for line in open(out)]
    for p, g in zip(prompts, got):
        seq = list(p)
        assert len(g) == 6
        for tok in g:
            assert tok == int(C.plain_logits(folder, seq)[-1].argmax())
            seq.append(tok)


def test_named_sizes_build():
    from mini_engine_amd.config.sizes import named_config
    cfg, full = named_config("venezen:tinyA")
    assert [layer.kind for layer in cfg.layers] == ["latent_attention"] * 2 and full == 2 and cfg.loop == (0, 0, 1)
    cfg, _ = named_config("venezen:0.6b", 8)
    model = build_model(cfg)
    assert len(model.order) == 8 and len(model.layers) == 6 and cfg.loop == (2, 4, 2)
    assert [c.layer for c in model.order] == [0, 1, 2, 3, 2, 3, 4, 5] and [c.add_start for c in model.order].index(True) == 4
