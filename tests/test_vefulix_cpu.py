"""Vefulix on the CPU: configuration, checkpoint layout, and the engine's bookkeeping for it (pages of a latent beside state
slots, models with only one of the two, batches, cuts, the scheduler) with the plain twins of the kernels in float32, against
the plain evaluation; each new twin against the plain function of its mechanism; and the plain evaluation with one mechanism
taken out, which must be far off (so that the random weights cannot hide a fault of that mechanism)."""
import copy
import json
import math

import pytest
import torch

import kernel_twins as twin
import plain_vefulix as P
import vefulix_cases as C
from mini_engine_amd.cache.manager import CacheManager
from mini_engine_amd.config.model_config import ConfigError, VefulixConfig, load_model_config
from mini_engine_amd.engine.runner import ModelRunner
from mini_engine_amd.kernels import ops
from mini_engine_amd.parts.norms import LayerNorm
from mini_engine_amd.registry import build_model
from mini_engine_amd.weights.loader import WeightError, load_model

CUTS = C.CUTS


@pytest.fixture(scope="module")
def vefulix_folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = C.make_folder(name, str(tmp_path_factory.mktemp(f"vefulix_{name}")))
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
        slots = slots if any(s is not None for s in model.cache_plan().state_needs) else 0
        manager = CacheManager(pages, C.PAGE[name], ModelRunner.windows_of(model), num_state_slots=slots, enable_prefix_caching=False)
        return ModelRunner(model, manager, self.dtype, self.device, 512, poison_cache=True), manager, folder


def test_config_reads_back_and_refuses_what_it_cannot_run(tmp_path):
    for name, raw in C.CONFIGS.items():
        cfg = VefulixConfig.from_dict(raw)
        assert VefulixConfig.from_dict(cfg.to_dict()) == cfg
        assert len(cfg.layers) == len(raw["layers"]) and cfg.vocab_size == raw["vocab"] and cfg.streams == raw["streams"]
    with open(tmp_path / "config.json", "w") as f:
        json.dump(C.CONFIGS["mix"], f)
    assert isinstance(load_model_config(str(tmp_path)), VefulixConfig)          # chosen by the file's architecture name
    alone = copy.deepcopy(C.CONFIGS["mix"])
    alone["layers"][0]["mixer"].pop("kv_heads")
    assert VefulixConfig.from_dict(alone).layers[0].mixer["kv_heads"] == 4      # absent: every head has a key of its own
    for spoil in (lambda c: c["layers"][0].update(type="delta2"),
                  lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
                  lambda c: c["layers"][0]["mixer"].pop("conv"),
                  lambda c: c["layers"][1]["mixer"].pop("q_rank"),
                  lambda c: c["layers"][1]["mixer"].update(scale=0.0),
                  lambda c: c["layers"][2]["mixer"].update(gate_cap=-1.0),
                  lambda c: c["layers"][1]["mlp"]["router"].update(top=9),
                  lambda c: c["layers"][1]["mlp"].update(kind="dense"),
                  lambda c: c["layers"][1]["mlp"].pop("expert"),
                  lambda c: c.pop("streams"),
                  lambda c: c.update(streams=0),
                  lambda c: c["norm"].pop("eps")):
        bad = copy.deepcopy(C.CONFIGS["mix"])
        spoil(bad)
        with pytest.raises(ConfigError):
            VefulixConfig.from_dict(bad)


def test_model_is_assembled_from_the_config(vefulix_folders, tmp_path):
    model = build_model(VefulixConfig.from_dict(C.CONFIGS["mix"]))
    plan = model.cache_plan()
    assert plan.call_group == [None, 0, None, 1]                                  # two ranks: two page groups
    assert plan.group_needs[0].tensors[0].shape[2] == 48 and plan.group_needs[1].tensors[0].shape[2] == 32      # ranks of 40 and 24 in steps of 16
    assert plan.state_needs[0].shape == (4 * 8 * 16 + (2 * 16 + 64) * 2,) and plan.state_needs[1] is None
    assert plan.state_needs[2].shape == (3 * 8 * 16 + 3 * 8 + 4,)                 # matrices, summed keys, maxima (in a whole step of 4)
    assert model.layers[3].feed_forward is None and model.layers[1].feed_forward.shared is None
    names = {src.name for sources in model.weight_sources.values() for src in sources}
    assert {"embed", "embed.norm", "embed.norm.b", "head", "final.norm.b", "l0.mix.q.conv", "l0.mix.A_log", "l0.mix.b", "l0.mix.a",
            "l0.mix.norm", "l0.hc1.in", "l0.hc2.mix", "l0.mlp.e7.gate", "l0.mlp.router.b", "l0.mlp.shared.down", "l1.mix.dq.norm", "l1.mix.uq",
            "l1.mix.dkv", "l1.mix.sink", "l2.mix.i.b", "l2.mix.f", "l2.mix.norm", "l3.norm1.b", "l3.hc1.out"} <= names
    assert not {"l3.hc2.in", "l3.norm2", "l1.mlp.shared.up"} & names
    # a checkpoint of another shape is refused as a whole
    from safetensors.torch import load_file, save_file
    folder = vefulix_folders("mix")
    tensors = load_file(folder + "/model.safetensors")
    tensors["l0.mix.q.conv"] = tensors["l0.mix.q.conv"][:, :2].contiguous()
    tensors["l9.extra"] = tensors.pop("l1.mix.sink")
    save_file(tensors, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(C.CONFIGS["mix"]))
    with pytest.raises(WeightError) as e:
        load_model(str(tmp_path), "cpu", torch.float32, 64)
    assert all(n in str(e.value) for n in ("l0.mix.q.conv", "l9.extra", "l1.mix.sink"))


# ---------------------------------------------------------------- each twin against the plain function of its mechanism

def _meta(q_lens, slots):
    cu = torch.tensor([0] + list(torch.tensor(q_lens).cumsum(0)), dtype=torch.int32)
    return cu, torch.tensor(slots, dtype=torch.int32)


CUT = ((0, 9), (9, 10), (10, 12), (12, 23))           # the state carries over the cuts


def test_matrix_memory_twins_in_steps_against_the_plain_loop():
    torch.manual_seed(0)
    T, H, N, Pv, width = 23, 3, 6, 5, 16
    m = {"heads": H, "dim": N, "vdim": Pv, "gate_cap": 3.0}
    h = torch.randn(T, width, dtype=torch.float64)
    w = {f"x.{n}": torch.randn(rows, width).double() for n, rows in (("q", H * N), ("k", H * N), ("v", H * Pv), ("g", H * Pv), ("i", H), ("f", H))}
    w |= {"x.i.b": torch.randn(H).double() * 2, "x.f.b": torch.randn(H).double() + 2, "x.norm": torch.rand(H * Pv).double() + 0.5, "x.o": torch.eye(H * Pv).double()}
    want = P.mlstm(h, w, "x.", m, 1e-5)
    row = lambda n: (h @ w["x." + n].T).float()
    state = torch.zeros(3, H * N * Pv + H * N + H)
    M, K = H * N * Pv, H * N
    got = []
    for lo, hi in CUT:
        cu, slots = _meta([hi - lo], [1])
        gates = ops.SoftGates(row("i")[lo:hi], row("f")[lo:hi], w["x.i.b"].float(), w["x.f.b"].float(), 3.0, state[:, M + K:], slots)
        reads = twin.linear_recurrence(row("q")[lo:hi], row("k")[lo:hi], row("v")[lo:hi], state[:, :M], slots, cu, [hi - lo], H, H, N, Pv,
                                       gates=gates, key_state=state[:, M:M + K])
        got.append(twin.memory_readout(reads, row("g")[lo:hi], w["x.norm"].float(), 1e-5, H, N ** -0.5, torch.float32))
    assert float((torch.cat(got).double() - want).abs().max()) < 1e-4 * float(want.abs().max())
    assert float(state[0].abs().max()) == 0 and float(state[2].abs().max()) == 0


def test_delta_twin_with_one_decay_per_head_against_the_plain_loop():
    torch.manual_seed(1)
    T, H, G, N, Pv, width = 23, 4, 2, 6, 5, 16
    m = {"heads": H, "kv_heads": G, "dim": N, "vdim": Pv, "conv": 3}
    h = torch.randn(T, width, dtype=torch.float64)
    w = {f"x.{n}": torch.randn(rows, width).double() for n, rows in (("q", G * N), ("k", G * N), ("v", H * Pv), ("g", H * Pv), ("a", H), ("b", H))}
    w |= {f"x.{n}.conv": torch.randn(rows, 3).double() for n, rows in (("q", G * N), ("k", G * N), ("v", H * Pv))}
    w |= {"x.A_log": torch.randn(H).double(), "x.dt_bias": torch.randn(H).double() - 2, "x.norm": torch.rand(Pv).double() + 0.5, "x.o": torch.eye(H * Pv).double()}
    want = P.delta(h, w, "x.", m, 1e-5)
    row = lambda n: (h @ w["x." + n].T).float()
    rows = torch.cat([row(n) for n in "qkv"], 1)
    taps = torch.cat([w[f"x.{n}.conv"] for n in "qkv"]).float()
    C_, M = rows.shape[1], H * N * Pv
    state = torch.zeros(3, M + C_ * 2)
    got = []
    for lo, hi in CUT:
        cu, slots = _meta([hi - lo], [1])
        x = twin.causal_conv(rows[lo:hi], taps, None, state[:, M:], slots, cu, [hi - lo])
        y = twin.decay_rows_recurrence(x[:, :G * N], x[:, G * N:2 * G * N], x[:, 2 * G * N:], row("a")[lo:hi], state[:, :M], slots, cu, [hi - lo],
                                       H, G, N, Pv, "delta_head", base=w["x.dt_bias"].float(), rate=torch.exp(w["x.A_log"]).float(),
                                       beta=row("b")[lo:hi], unit_eps=1e-6, q_scale=N ** -0.5)
        got.append(twin.gated_rms_norm(y, row("g")[lo:hi], w["x.norm"].float().repeat(H), 1e-5, H, "silu_behind", torch.float32))
    assert float((torch.cat(got).double() - want).abs().max()) < 1e-4 * float(want.abs().max())
    assert float(state[0].abs().max()) == 0 and float(state[2].abs().max()) == 0


def test_latent_twins_with_a_query_latent_and_sinks_against_the_plain_heads():
    """One key that stands out for a query far away, at a page's border: leaving it out shows."""
    torch.manual_seed(5)
    T, H, dn, nv, R, Rq, width, page = 30, 3, 6, 5, 10, 7, 12, 4
    m = {"heads": H, "dim": dn, "vdim": nv, "q_rank": Rq, "kv_rank": R, "scale": 0.9}
    h = torch.randn(T, width, dtype=torch.float64)
    w = {f"x.{n}": torch.randn(*s).double() for n, s in (("dq", (Rq, width)), ("uq", (H * dn, Rq)), ("dkv", (R, width)), ("uk", (H * dn, R)), ("uv", (H * nv, R)))}
    w |= {"x.dq.norm": torch.rand(Rq).double() + 0.5, "x.dkv.norm": torch.rand(R).double() + 0.5, "x.sink": torch.tensor([1.0, 4.0, -1.0]).double(),
          "x.o": torch.eye(H * nv).double()}
    # head 0: the last query points at the key of position 3, the last of the first page
    c = (P.unit_rms(h @ w["x.dkv"].T, 1e-5) * w["x.dkv.norm"])[3]
    q = ((P.unit_rms(h @ w["x.dq"].T, 1e-5) * w["x.dq.norm"]) @ w["x.uq"].T).view(T, H, dn)[29, 0]
    w["x.uk"][:dn] += 3.0 * torch.outer(q, c) / (c @ c)
    want = P.latent_attention(h, w, "x.", m, 1e-5)
    D = 16
    rows = torch.cat((h @ w["x.dq"].T, h @ w["x.dkv"].T), 1).float()
    kc, vc = torch.full((9, 1, page, D), float("nan")), torch.full((9, 1, D, page), float("nan"))
    pos = torch.arange(T, dtype=torch.int32)
    qa, cq = twin.latent_prepare(rows, 0, Rq, H, 0, 0, R, D, w["x.dkv.norm"].float(), 1e-5, None, pos, pos, kc, vc, page,
                                 query_latent=(0, w["x.dq.norm"].float()))
    q = cq @ w["x.uq"].float().T
    uk_t = w["x.uk"].float().view(H, dn, R).transpose(1, 2).contiguous()
    twin.heads_linear(q.view(T, H, dn), uk_t, qa.view(T, H, D)[:, :, :R])
    bt = torch.arange(9, dtype=torch.int32)[None]
    o = twin.paged_attention(qa, kc, vc, page, bt, torch.tensor([T], dtype=torch.int32), torch.zeros(T, dtype=torch.int32), pos,
                             torch.tensor([0, T], dtype=torch.int32), 0, 0, 0.9, None, H, 1, D, max_prefill_context=T, sinks=w["x.sink"].float())
    heads = torch.empty(T, H * nv)
    twin.heads_linear(o.view(T, H, D)[:, :, :R], w["x.uv"].float().view(H, nv, R), heads.view(T, H, nv))
    assert float((heads.double() - want).abs().max()) < 2e-5 * float(want.abs().max())
    other = h.clone()
    other[3] = torch.randn(width).double()
    moved = P.latent_attention(other, w, "x.", m, 1e-5)[29] - want[29]
    assert float(moved.abs().max()) > 1e-2 * float(want.abs().max())


def test_stream_twin_against_the_plain_streams():
    torch.manual_seed(7)
    T, S, n = 6, 3, 10
    w = {"x.in": torch.randn(S).double(), "x.out": torch.randn(S).double(), "x.mix": torch.randn(S, S).double(), "y.in": torch.randn(S).double(),
         "n": torch.rand(n).double() + 0.5, "n.b": torch.randn(n).double()}
    x, a, b = torch.randn(T, S, n).double(), torch.randn(2, T, n), torch.randn(T, n)
    old = x.permute(1, 0, 2)
    new = P.write_streams(old, (a.sum(0) + b).double(), w, "x.")
    want = P.layer_norm(P.read_streams(new, w, "y."), w, "n", 1e-3)
    f = {k: v.float() for k, v in w.items()}
    norm = (f["n"], f["n.b"], 1e-3, True)
    got_new, got = twin.stream_mix_norm(x.float(), S, [a, b], f["x.mix"], f["x.out"], f["y.in"], norm, torch.float32)
    assert torch.allclose(got_new.double(), new.permute(1, 0, 2), atol=1e-5) and torch.allclose(got.double(), want, atol=1e-5)
    turned = P.write_streams(old, (a.sum(0) + b).double(), dict(w, **{"x.mix": w["x.mix"].T.contiguous()}), "x.")
    assert float((turned - new).abs().max()) > 0.1                     # from and to are not alike
    rows = torch.tensor([4, 0], dtype=torch.int32)
    none, picked = twin.stream_mix_norm(x.float(), S, [a, b], f["x.mix"], f["x.out"], None, norm, torch.float32, rows=rows, keep=False)
    assert none is None and torch.allclose(picked.double(), P.layer_norm(new.sum(0), w, "n", 1e-3)[[4, 0]], atol=1e-5)
    # rows that all streams share
    _, shared = twin.stream_mix_norm(b, S, [], None, None, f["y.in"], norm, torch.float32, keep=False)
    assert torch.allclose(shared.double(), P.layer_norm(P.read_streams(torch.stack([b.double()] * S), w, "y."), w, "n", 1e-3), atol=1e-5)


def test_layer_norm_part_on_its_own(plain_backend):
    """The norm as any block may use it: starting a stream, adding to one, adding partial sums."""
    torch.manual_seed(8)
    part = LayerNorm(12, 1e-4)
    part.set_param("weight", torch.rand(12) + 0.5)
    part.set_param("bias", torch.randn(12))
    part.finalize("cpu", torch.float32, 8)
    ref = lambda r: torch.nn.functional.layer_norm(r, (12,), part.weight, part.bias, 1e-4)
    x, r, p = torch.randn(5, 12), torch.randn(5, 12), torch.randn(3, 5, 12)
    y, stream = part.forward(x, None)
    assert torch.allclose(y, ref(x), atol=1e-6) and torch.equal(stream, x)
    y, stream = part.forward(x, r)
    assert torch.allclose(stream, x + r) and torch.allclose(y, ref(x + r), atol=1e-6)
    y, stream = part.forward(p, r)
    assert torch.allclose(stream, p.sum(0) + r, atol=1e-6) and torch.allclose(y, ref(p.sum(0) + r), atol=1e-5)


def test_router_twin_that_chooses_by_its_logits():
    torch.manual_seed(3)
    T, E, n = 50, 12, 10
    x, router, bias = torch.randn(T, n), torch.randn(E, n), torch.randn(E) * 2
    for top in (1, 3, 12):
        ids, weights = P.choose_experts((x @ router.T + bias).double(), top)
        got_ids, got_w = twin.moe_route(x, router, top, 1, 1, ops.RouteRule("chosen", bias=bias))
        assert torch.equal(got_ids.long(), ids) and torch.allclose(got_w.double(), weights, atol=1e-6)
        assert torch.allclose(got_w.sum(-1), torch.ones(T))
    # logits so far apart that a softmax over all experts would lose the smaller ones
    far = twin.moe_route(torch.eye(1), torch.tensor([[0.0], [-200.0], [-300.0]]), 3, 1, 1, ops.RouteRule("chosen"))
    assert far[0].tolist() == [[0, 1, 2]]


# ---------------------------------------------------------------- a mechanism left out must show

def _zero(name):
    return lambda cfg, w: w.update({name: torch.zeros_like(w[name])})


def _one(name):
    return lambda cfg, w: w.update({name: torch.ones_like(w[name])})


SPOILS = {
    "embedding_norm_bias": _zero("embed.norm.b"), "norm1_bias": _zero("l1.norm1.b"), "norm2_bias": _zero("l0.norm2.b"), "final_norm_bias": _zero("final.norm.b"),
    "mean": lambda cfg, w: w.update({"embed": w["embed"] + 1.0, "?": None}),
    "read_shares": lambda cfg, w: w.update({"l1.hc1.in": torch.full_like(w["l1.hc1.in"], 0.5)}),
    "write_shares": _one("l2.hc2.out"), "mix": lambda cfg, w: w.update({"l2.hc1.mix": torch.eye(2)}),
    "mix_turned": lambda cfg, w: w.update({"l1.hc2.mix": w["l1.hc2.mix"].T.contiguous()}),
    "taps_turned": lambda cfg, w: w.update({"l0.mix.k.conv": w["l0.mix.k.conv"].flip(1).contiguous()}),
    "value_conv": lambda cfg, w: w.update({"l0.mix.v.conv": w["l0.mix.v.conv"] * torch.tensor([0.0, 0.0, 1.0])}),
    "write_strength": _zero("l0.mix.b"), "decay_rate": _zero("l0.mix.A_log"), "decay_bias": _zero("l0.mix.dt_bias"), "decay": _zero("l0.mix.a"),
    "delta_norm": _one("l0.mix.norm"), "delta_gate": _one("l0.mix.g"),
    "shared_keys": lambda cfg, w: w.update({n: w[n].roll(8, 0) for n in ("l0.mix.k", "l0.mix.k.conv")}),
    "input_bias": _zero("l2.mix.i.b"), "forget_bias": _zero("l2.mix.f.b"), "gate_cap": lambda cfg, w: cfg["layers"][2]["mixer"].update(gate_cap=50.0),
    "input_gate": _zero("l2.mix.i"), "memory_norm": _one("l2.mix.norm"), "memory_gate": _zero("l2.mix.g"),
    "sink": lambda cfg, w: w.update({"l1.mix.sink": w["l1.mix.sink"] - 30.0}), "query_latent_norm": _one("l1.mix.dq.norm"),
    "latent_norm": _one("l1.mix.dkv.norm"), "score_scale": lambda cfg, w: cfg["layers"][3]["mixer"].update(scale=0.6),
    "router_bias": _zero("l0.mlp.router.b"), "top": lambda cfg, w: cfg["layers"][2]["mlp"]["router"].update(top=2),
    "shared_expert": lambda cfg, w: cfg["layers"][0]["mlp"].pop("shared"), "softcap": lambda cfg, w: cfg.pop("logit_softcap"),
}


@pytest.mark.parametrize("spoil", [*SPOILS, "memory_floor", "softmax_over_all"])
def test_the_weights_show_a_mechanism_that_is_left_out(vefulix_folders, monkeypatch, spoil):
    folder = vefulix_folders("mix")
    cfg, w = P.read_folder(folder)
    ids = C.random_ids(40, 101, 5)
    ref = P.logits(cfg, w, ids)
    cfg, w = copy.deepcopy(cfg), dict(w)
    if spoil == "memory_floor":              # the scale of keys and queries shows in the output only through the floor
        w["l2.mix.q"] = w["l2.mix.q"] * 0.25
    elif spoil == "softmax_over_all":
        monkeypatch.setattr(P, "choose_experts", lambda z, top: (z.topk(top, -1).indices, torch.softmax(z, -1).topk(top, -1).values))
    else:
        SPOILS[spoil](cfg, w)
        w.pop("?", None)
    off = P.logits(cfg, w, ids)
    moved = float((off - ref).abs().max() / ref.abs().max())
    if spoil == "mean":                        # a constant on every embedding element: the mean is taken off, nothing may move
        assert moved < 3e-2
        return
    if spoil == "memory_floor":                # every head's output is normed: without the floor a scale of q would change nothing
        assert moved > 1e-3
        return
    assert moved > 2e-3, f"leaving out {spoil} hardly shows in the logits: {moved:.2g}"


def test_keys_far_away_show_in_the_logits(vefulix_folders):
    """In the model of latent layers alone, an early token that some later query asks for moves that query's logits hundreds of
    positions on; so a lost page or key cannot hide."""
    cfg, w = P.read_folder(vefulix_folders("pages"))
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
def test_every_layer(vefulix_folders, plain_backend, name):
    C.layers_one_by_one(Env(vefulix_folders), name)


@pytest.mark.parametrize("name", C.SMALL)
@pytest.mark.parametrize("case", CUTS.ALL, ids=lambda c: c.__name__)
def test_cuts(vefulix_folders, plain_backend, case, name):
    case(Env(vefulix_folders), name)


@pytest.mark.parametrize("name", ["pages", "mix"])
def test_long_prompts(vefulix_folders, plain_backend, name):
    CUTS.long_prompt(Env(vefulix_folders), name)


@pytest.mark.parametrize("name", ["mix", "odd", "pages"])
def test_greedy_generation_through_the_scheduler(vefulix_folders, plain_backend, name):
    CUTS.greedy_through_the_engine("cpu", "float32", name, vefulix_folders(name), exact=True)


def test_streams_behind_a_block_of_another_kind(plain_backend):
    """A layer with several streams may follow an ordinary one: what that one has left is added, and every stream starts there."""
    from mini_engine_amd.parts.base import make_part
    torch.manual_seed(4)
    n = 8
    norm = lambda: make_part("norm", "layer", size=n, eps=1e-5)

    class Add(torch.nn.Module):
        def forward(self, x, *a):
            return 2.0 * x

    block = make_part("block", "hyper_connected", streams=2, norm1=norm(), mixer=make_part("mixer", "mlstm", hidden_size=n, num_heads=1, key_dim=4,
                                                                                          value_dim=4, gate_cap=4.0, norm_eps=1e-5))
    block.mixer = Add()
    block.read1, block.out1, block.mix1 = torch.tensor([0.5, 1.0]), torch.tensor([1.0, -1.0]), torch.tensor([[0.5, 0.2], [0.1, 0.9]])
    block.norm1.weight, block.norm1.bias = torch.rand(n), torch.rand(n)
    h, residual = torch.randn(3, n), torch.randn(3, n)
    out, streams = block.forward(h, residual, None, None, None)
    x = h + residual
    y = 2.0 * torch.nn.functional.layer_norm(1.5 * x, (n,), block.norm1.weight, block.norm1.bias, 1e-5)
    assert torch.allclose(out.settle(streams), (0.6 + 1.1) * x + 0.0 * y, atol=1e-5)
    assert torch.allclose(out.normed_rows(streams, block.norm1, torch.tensor([2], dtype=torch.int32)),
                          torch.nn.functional.layer_norm(1.7 * x, (n,), block.norm1.weight, block.norm1.bias, 1e-5)[2:], atol=1e-5)


def test_command_line_on_a_folder_of_this_design(vefulix_folders, plain_backend, tmp_path):
    """`python -m mini_engine_amd.cli --model DIR`: the folder's config picks the model class; prompts in, greedy tokens out."""
    from mini_engine_amd import cli
    import helpers
    folder = vefulix_folders("mix")
    prompts = [helpers.random_ids(n, 101, 950 + n) for n in (3, 19, 41)]
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
    cfg, full = named_config("vefulix:tinyA")
    model = build_model(cfg)
    assert [layer.kind for layer in cfg.layers] == ["delta", "latent_attention"] and full == 2 and model.layers[1].feed_forward.num_experts == 32
    cfg, _ = named_config("vefulix:0.6b", 8)
    plan = build_model(cfg).cache_plan()
    assert plan.call_writes == [False, True] * 4 and math.prod(plan.state_needs[2].shape) == 4 * 128 * 256 + 4 * 128 + 4


def test_launch_rule_of_the_delta_rule_with_one_decay_per_head():
    """Sixteen lanes to a column while the waves run in one round (a wave keeps fewer values in LDS than with a decay per row);
    single tokens beside long portions do not count as chains."""
    from mini_engine_amd.kernels import ops
    rule = lambda lens, one: ops.decay_row_groups(len(lens), 8, 128, 128, max(lens), sum(lens), one)
    assert rule([700] * 8, True) == (16, True) and rule([700] * 8, False) == (4, True)
    assert rule([700] * 4, False) == (16, True) and rule([700] * 16, True) == (4, True)
    assert rule([700] * 7 + [1] * 40, True) == (16, True)
    assert rule([1] * 64, True) == (4, False)
