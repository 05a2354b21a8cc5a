"""Vefulix on the GPU: each new kernel (and each new form of an older one) against its plain twin at sizes of its own, then
every layer, the engine's cuts, batches, slot and page reuse and long decoding in float32 and bfloat16 against the plain
evaluation, real layer sizes, decode steps replayed as graphs, greedy generation through the scheduler, and the trace program
on folders of this design."""
import pytest
import torch

import helpers
import kernel_twins as twin
import test_trace_run as TR
import vefulix_cases as C
from mini_engine_amd.cache.manager import CacheManager
from mini_engine_amd.engine.runner import ModelRunner
from mini_engine_amd.kernels import ops
from mini_engine_amd.parts.rotary import RotaryEmbedding
from mini_engine_amd.weights.loader import load_model

pytestmark = pytest.mark.gpu
DEV = "cuda"
TOL = {torch.float32: 5e-5, torch.bfloat16: 2.5e-1}    # widths of 24-64 make bfloat16 noisy: single rows far, the mean near
MEAN_TOL = {torch.float32: 5e-5, torch.bfloat16: 4e-2}
CUTS = C.CUTS
DTYPES = [torch.float32, torch.bfloat16]


def hip():
    return ops.HipBackend()


def close(a, b, tol):
    a, b = a.double().cpu(), b.double().cpu()
    assert a.shape == b.shape and torch.isfinite(a).all()
    err = float((a - b).abs().max() / b.abs().max().clamp_min(1e-30))
    assert err <= tol, f"relative error {err:.3g} > {tol:g}"


@pytest.fixture(scope="module")
def vefulix_folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = C.make_folder(name, str(tmp_path_factory.mktemp(f"vefulix_{name}")))
        return made[name]

    return get


def _meta(q_lens, slots):
    cu = torch.tensor([0] + list(torch.tensor(q_lens).cumsum(0)), dtype=torch.int32, device=DEV)
    return cu, torch.tensor(slots, dtype=torch.int32, device=DEV)


def _cpu(t):
    return t.cpu() if torch.is_tensor(t) else t


# ------------------------------------------------------------------ kernels against their twins

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 6, 7, 8, 11])
@pytest.mark.parametrize("T,n", [(5, 64), (37, 50), (600, 132), (3, 4100), (1, 3)])
def test_stream_mix_norm(dtype, S, T, n):
    """Mixed and not, with and without terms, a layer norm, an RMS norm and none, chosen rows, rows that all streams share."""
    torch.manual_seed(S * n + T)
    f = lambda *s: torch.randn(*s, device=DEV)
    x, a, b, c = f(T, S, n), f(3, T, n), f(T, n).to(dtype), f(T, n)
    mix, out, read, w, bias = f(S, S), f(S), f(S), f(n), f(n)
    rows = torch.randint(0, T, (7,), device=DEV, dtype=torch.int32)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    for terms, m, o, r, norm, pick, streams in (
            ([a, b], mix, out, read, (w, bias, 1e-5, True), None, x), ([b], mix, out, read, (w, None, 1e-5, False), None, x),
            ([], None, None, read, (w, bias, 1e-5, True), None, x), ([a], None, None, None, (w, bias, 1e-5, True), None, x),
            ([a, b, c, b], mix, out, None, (w, bias, 1e-3, True), rows, x), ([a, b], mix, out, None, None, None, x),
            ([b], mix, out, read, (w, bias, 1e-5, True), None, c), ([], None, None, read, (w, bias, 1e-5, True), None, b),
            ([], None, None, None, (w, bias, 1e-5, True), rows, b)):
        got_new, got = hip().stream_mix_norm(streams, S, terms, m, o, r, norm, dtype, rows=pick)
        want_new, want = twin.stream_mix_norm(streams.cpu(), S, [t.cpu() for t in terms], _cpu(m), _cpu(o), _cpu(r),
                                              None if norm is None else tuple(_cpu(t) for t in norm), dtype, rows=_cpu(pick))
        close(got_new, want_new, 2e-6 * S)
        close(got, want, tol)
        assert hip().stream_mix_norm(streams, S, terms, m, o, r, norm, dtype, rows=pick, keep=False)[0] is None


SIZES = [(3, 8, 16), (2, 10, 14), (4, 128, 256), (1, 200, 7), (2, 64, 64), (5, 48, 100)]


@pytest.mark.parametrize("spans", [None, (16, 6), (64, 2)], ids=["rule", "spans16", "spans64"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,N,P", SIZES)
def test_matrix_memory(monkeypatch, dtype, H, N, P, spans):
    """Gates, recurrence with summed keys and readout over requests of unequal lengths from states of their own, against the
    token-by-token twin; then one request in portions and single tokens gives what it gives whole."""
    if spans:
        monkeypatch.setattr(ops, "recurrence_spans", lambda *a: spans)
    torch.manual_seed(H * N + P)
    q_lens = [1, 90, 2, 70]
    cu, slots = _meta(q_lens, [2, 0, 4, 1])
    T, M, K = sum(q_lens), H * N * P, H * N
    width = 2 * K + 2 * H * P + 2 * H
    rows = torch.randn(T, (width + 7) // 8 * 8 + 8, device=DEV).to(dtype)
    rows[:, 2 * K + 2 * H * P:] *= 3
    rows[:, : 2 * K] *= 0.5
    bi, bf, w = torch.randn(H, device=DEV), torch.randn(H, device=DEV) + 2, torch.rand(H * P, device=DEV) + 0.5
    pad = -(M + K + H) % 4
    full = torch.randn(6, M + K + H + pad, device=DEV)

    def run(B, rows, state, slots, cu, lens):
        at = 2 * K + 2 * H * P
        gates = ops.SoftGates(rows[:, at:at + H], rows[:, at + H:at + 2 * H], bi.to(rows.device), bf.to(rows.device), 4.0, state[:, M + K:M + K + H], slots)
        reads = B.linear_recurrence(rows[:, :K], rows[:, K:2 * K], rows[:, 2 * K:2 * K + H * P], state[:, :M], slots, cu, lens, H, H, N, P,
                                    gates=gates, key_state=state[:, M:M + K])
        return B.memory_readout(reads, rows[:, 2 * K + H * P:at], w.to(rows.device), 1e-5, H, N ** -0.5, dtype)

    st_h, st_c = full.clone(), full.cpu().clone()
    got = run(hip(), rows, st_h, slots, cu, q_lens)
    want = run(twin, rows.cpu(), st_c, slots.cpu(), cu.cpu(), q_lens)
    close(got, want, 2e-2 if dtype == torch.bfloat16 else 5e-5)
    close(st_h, st_c, 2e-5)
    assert torch.equal(st_h[3], full[3]) and torch.equal(st_h[5], full[5])
    st2, parts = full.clone(), []
    for lo, hi in ((1, 40), (40, 41), (41, 42), (42, 44), (44, 91)):
        cu1, slots1 = _meta([hi - lo], [0])
        parts.append(run(hip(), rows[lo:hi], st2, slots1, cu1, [hi - lo]))
    close(torch.cat(parts), got[1:91], 2e-2 if dtype == torch.bfloat16 else 2e-5)
    close(st2[0], st_h[0], 1e-5)
    # a step of single tokens for several requests at once
    cu3, slots3 = _meta([1, 1, 1], [5, 3, 1])
    st3, st3c = st_h.clone(), st_h.cpu().clone()
    close(run(hip(), rows[:3], st3, slots3, cu3, [1, 1, 1]), run(twin, rows[:3].cpu(), st3c, slots3.cpu(), cu3.cpu(), [1, 1, 1]),
          2e-2 if dtype == torch.bfloat16 else 5e-5)
    close(st3, st3c, 2e-5)


@pytest.mark.parametrize("groups", [None, (1, False), (4, False), (4, True), (16, True)],
                         ids=["rule", "one-lane", "four-lanes", "four-lanes-prepared", "sixteen-lanes-prepared"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,P", [(4, 2, 8, 16), (6, 2, 10, 14), (4, 4, 128, 128), (3, 1, 200, 7), (2, 1, 64, 64), (1, 1, 96, 80)])
def test_delta_rule_with_one_decay_per_head(monkeypatch, dtype, H, G, N, P, groups):
    """Requests of unequal lengths from states of their own, against the token-by-token twin; then one request cut in portions
    gives what it gives whole."""
    if groups:
        if groups[0] == 1 and N > 64:
            pytest.skip("a lane keeps up to 64 rows")
        monkeypatch.setattr(ops, "decay_row_groups", lambda *a: groups)
    torch.manual_seed(H * N + P)
    q_lens = [1, 130, 2, 17]
    cu, slots = _meta(q_lens, [2, 0, 4, 1])
    T, qk, M = sum(q_lens), G * N, H * N * P
    rows = torch.randn(T, 2 * qk + H * P + 2 * H + 3, device=DEV).to(dtype)
    cols = lambda r: (r[:, :qk], r[:, qk:2 * qk], r[:, 2 * qk:2 * qk + H * P], r[:, 2 * qk + H * P:2 * qk + H * P + H])
    kw = dict(base=torch.randn(H, device=DEV) - 1, rate=torch.rand(H, device=DEV) + 0.2, unit_eps=1e-6, q_scale=N ** -0.5)
    beta = lambda r: r[:, 2 * qk + H * P + H:2 * qk + H * P + 2 * H]
    full = torch.randn(6, 4 + M, device=DEV)
    st_h, st_c = full.clone(), full.cpu().clone()
    got = hip().decay_rows_recurrence(*cols(rows), st_h[:, 4:], slots, cu, q_lens, H, G, N, P, "delta_head", beta=beta(rows), **kw)
    want = twin.decay_rows_recurrence(*cols(rows.cpu()), st_c[:, 4:], slots.cpu(), cu.cpu(), q_lens, H, G, N, P, "delta_head", beta=beta(rows.cpu()),
                                      **{n: _cpu(t) for n, t in kw.items()})
    close(got, want, 2e-5)
    close(st_h, st_c, 2e-5)
    assert torch.equal(st_h[:, :4], full[:, :4]) and torch.equal(st_h[3], full[3]) and torch.equal(st_h[5], full[5])
    st2, parts = full.clone(), []
    for lo, hi in ((1, 40), (40, 41), (41, 43), (43, 131)):
        cu1, slots1 = _meta([hi - lo], [0])
        r = rows[lo:hi]
        parts.append(hip().decay_rows_recurrence(*cols(r), st2[:, 4:], slots1, cu1, [hi - lo], H, G, N, P, "delta_head", beta=beta(r), **kw))
    close(torch.cat(parts), got[1:131], 1e-5)
    close(st2[0], st_h[0], 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dn,dr,nv,R,Rq,page", [(5, 24, 0, 40, 72, 40, 16), (3, 12, 6, 10, 20, 13, 8), (16, 128, 0, 128, 256, 384, 16), (1, 8, 8, 8, 16, 5, 4)])
def test_latent_prepare_with_a_latent_for_the_queries(dtype, H, dn, dr, nv, R, Rq, page):
    """Both latents' norms and the page writes in one pass, with and without a rotating part, against the twin."""
    torch.manual_seed(H + R)
    T, D = 37, -(-(R + dr) // 16) * 16
    table = None
    if dr:
        enc = RotaryEmbedding(dr, 5000.0, interleaved=True, exact_angles=True)
        enc.finalize(DEV, dtype, 512)
        table = enc.table
    rows = torch.randn(T, Rq + R + dr + 5, device=DEV).to(dtype)
    w, wq = torch.rand(R, device=DEV) + 0.5, torch.rand(Rq, device=DEV) + 0.5
    pos = torch.randint(0, 512, (T,), device=DEV, dtype=torch.int32)
    slots = torch.randperm(10 * page, device=DEV)[:T].to(torch.int32)
    slots[5] = -1
    kc = torch.full((11, 1, page, D), 7.0, device=DEV, dtype=dtype)
    vc = torch.full((11, 1, D, page), 7.0, device=DEV, dtype=dtype)
    kc2, vc2 = kc.cpu().clone(), vc.cpu().clone()
    args = (rows, 0, Rq, 0 if dr else H, 0, dr, R, D, w, 1e-5, table, pos, slots, kc, vc, page)
    qa, cq = hip().latent_prepare(*args, query_latent=(0, wq))
    args2 = tuple(_cpu(a) for a in args[:13]) + (kc2, vc2, page)
    qa2, cq2 = twin.latent_prepare(*args2, query_latent=(0, wq.cpu()))
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    close(cq, cq2, tol)
    close(kc, kc2, tol)
    close(vc, vc2, tol)
    if not dr:
        assert torch.equal(qa.view(T, H, D)[:, :, R:].cpu(), torch.zeros(T, H, D - R, dtype=dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,E,n,top", [(50, 12, 40, 3), (3, 10, 256, 3), (200, 32, 64, 4), (7, 6, 36, 6), (33, 4, 16, 1), (64, 64, 128, 6), (20, 100, 24, 64)])
def test_router_that_chooses_by_its_logits(dtype, T, E, n, top):
    """The choice and the weights (a softmax over the chosen logits alone) against the twin, through the kernel of its own and,
    for few tokens, inside the kernel that orders the pairs."""
    torch.manual_seed(T + E)
    x = torch.randn(T, n, device=DEV).to(dtype)
    router = torch.randn(E, n, device=DEV) * 3.0 * n ** -0.5
    rule = ops.RouteRule("chosen", bias=torch.randn(E, device=DEV) * 2)
    ids, weights = hip().moe_route(x, router, top, 1, 1, rule)
    want_ids, want_w = twin.moe_route(x.cpu(), router.cpu(), top, 1, 1, ops.RouteRule("chosen", bias=rule.bias.cpu()))
    z = x.float() @ router.t() + rule.bias
    gap = z.sort(-1).values.diff(dim=-1)
    sure = gap[:, max(0, E - top - 1):].amin(-1).cpu() > 1e-4 if E > 1 else torch.ones(T, dtype=torch.bool)
    assert sure.float().mean() > 0.6
    assert torch.equal(ids.cpu()[sure], want_ids[sure])
    close(weights.cpu()[sure], want_w[sure], 1e-5)
    F, hidden = 24, 40
    gu = (torch.randn(E, 2 * F, n, device=DEV) * 0.2).to(dtype)
    down = (torch.randn(E, hidden, F, device=DEV) * 0.2).to(dtype)
    got = hip().route_and_run_experts(x, router, top, 1, 1, gu, down, rule=rule)
    want = twin.routed_experts(x.cpu(), ids.cpu(), weights.cpu(), gu.cpu(), down.cpu())
    close(got.sum(0), want.sum(0), 3e-2 if dtype == torch.bfloat16 else 2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["silu_before", "sigmoid_behind", "silu_behind"])
@pytest.mark.parametrize("groups,per", [(3, 16), (2, 100), (5, 128), (4, 256), (2, 300), (2, 1000), (3, 2050), (4, 6)])
def test_gated_norm_per_group(dtype, kind, groups, per):
    torch.manual_seed(groups * per)
    T, n = 13, groups * per
    y, wide, w = torch.randn(2, T, n, device=DEV), torch.randn(T, n + 12, device=DEV).to(dtype), torch.rand(n, device=DEV) + 0.5
    for at in (4, 3):                              # gate rows that start at a whole piece, and not
        gate = wide[:, at:at + n]
        close(hip().gated_rms_norm(y, gate, w, 1e-5, groups, kind, dtype), twin.gated_rms_norm(y.cpu(), gate.cpu(), w.cpu(), 1e-5, groups, kind, dtype),
              1e-2 if dtype == torch.bfloat16 else 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,H,page", [(32, 3, 8), (256, 16, 16), (80, 5, 16), (16, 1, 4)])
def test_sinks_over_one_shared_key_head_with_a_far_key_that_stands_out(dtype, D, H, page):
    """One key/value head under all query heads, sinks of every size, requests in prompts of several lengths and decoding: the
    key that a query asks for lies far away at a page's border, and one score stands out."""
    torch.manual_seed(D + H)
    lens, news = [300, 41, 700, 18], [1, 1, 90, 18]
    sinks = torch.linspace(-3.0, 12.0, H, device=DEV)
    MB = max(-(-n // page) for n in lens)
    perm = torch.randperm(len(lens) * MB)
    bt = perm.view(len(lens), MB).to(torch.int32).to(DEV)
    kc = torch.randn(len(lens) * MB + 1, 1, page, D, device=DEV).to(dtype) * 0.5
    vc = torch.randn(len(lens) * MB + 1, 1, D, page, device=DEV).to(dtype)
    T = sum(news)
    q = torch.randn(T, H * D, device=DEV).to(dtype)
    pos = torch.cat([torch.arange(n - k, n) for n, k in zip(lens, news)]).to(torch.int32).to(DEV)
    seq = torch.repeat_interleave(torch.arange(len(lens)), torch.tensor(news)).to(torch.int32).to(DEV)
    last = torch.tensor(news).cumsum(0) - 1
    for r, n in enumerate(lens):                   # each request's last query, head 0, asks for the key one before its first page border
        kc[bt[r, 0], 0, page - 1] = (q[last[r], :D].float() * 6.0 * D ** -0.5).to(dtype)
    ctx = torch.tensor(lens, dtype=torch.int32, device=DEV)
    cu = torch.tensor([0, 90, 108], dtype=torch.int32, device=DEV)
    args = lambda dev: [t.to(dev) if torch.is_tensor(t) else t for t in (q, kc, vc, page, bt, ctx, seq, pos, cu, 2, 300, D ** -0.5, None, H, 1, D)]
    got = hip().paged_attention(*args(DEV), max_prefill_context=700, sinks=sinks)
    want = twin.paged_attention(*[a.float() if torch.is_tensor(a) and a.is_floating_point() else a for a in args("cpu")], max_prefill_context=700, sinks=sinks.cpu())
    close(got, want, 2e-2 if dtype == torch.bfloat16 else 2e-5)
    without = twin.paged_attention(*[a.float() if torch.is_tensor(a) and a.is_floating_point() else a for a in args("cpu")], max_prefill_context=700)
    assert float((without - want).abs().max()) > 0.03 * float(want.abs().max())
    for forced in ({"decode_as_prefill": True}, {"force_simple": True}):
        close(hip().paged_attention(*args(DEV), max_prefill_context=700, sinks=sinks, **forced), want, 2e-2 if dtype == torch.bfloat16 else 2e-5)


# ------------------------------------------------------------------ the engine against the plain evaluation

def as_held(name, dtype):
    """The configuration that a dtype is held to the tolerance on, row by row: in bfloat16 the one whose tokens take every expert (a
    choice between two close logits may fall otherwise there; what is chosen is held by the router's own test and in the mean)."""
    return name if dtype in (torch.float32, "float32") else name + "-all"


class Env:
    device = DEV

    def __init__(self, folders, dtype, graphs=False):
        self.folders, self.dtype, self.tol, self.mean_tol, self.graphs, self.models = folders, dtype, TOL[dtype], MEAN_TOL[dtype], graphs, {}

    def runner(self, name, pages, slots):
        folder = self.folders(name)
        if name not in self.models:
            self.models[name] = load_model(folder, self.device, self.dtype, 1024)
        model = self.models[name]
        slots = slots if any(s is not None for s in model.cache_plan().state_needs) else 0
        manager = CacheManager(pages, C.PAGE[name], ModelRunner.windows_of(model), num_state_slots=slots, enable_prefix_caching=False)
        options = dict(use_graphs=True, mixed_graphs_after=1) if self.graphs else {}
        return ModelRunner(model, manager, self.dtype, self.device, 1024, poison_cache=True, **options), manager, folder


@pytest.fixture(scope="module", params=DTYPES, ids=["float32", "bfloat16"])
def env(request, vefulix_folders):
    return Env(vefulix_folders, request.param)


@pytest.mark.parametrize("name", C.SMALL)
def test_every_layer(env, name):
    C.layers_one_by_one(env, as_held(name, env.dtype))


@pytest.mark.parametrize("name", C.SMALL)
@pytest.mark.parametrize("case", CUTS.ALL, ids=lambda c: c.__name__)
def test_cuts(env, case, name):
    case(env, as_held(name, env.dtype))


@pytest.mark.parametrize("name", ["pages", "mix", "odd"])
def test_long_prompts(env, name):
    CUTS.long_prompt(env, as_held(name, env.dtype))


def test_real_layer_sizes(vefulix_folders):
    C.real_sizes(Env(vefulix_folders, torch.float32), Env(vefulix_folders, torch.bfloat16))


def test_real_layer_sizes_with_a_choice_of_experts(vefulix_folders):
    C.real_sizes(Env(vefulix_folders, torch.float32), Env(vefulix_folders, torch.bfloat16), "routed", every_row=False)


@pytest.mark.parametrize("dtype", DTYPES, ids=["float32", "bfloat16"])
@pytest.mark.parametrize("case", [CUTS.token_by_token, CUTS.long_decode, CUTS.batch_against_alone], ids=lambda c: c.__name__)
def test_cuts_through_captured_steps(vefulix_folders, case, dtype):
    """The same with decode steps (and small steps that come up again) replayed as graphs: state slots travel with the
    step's metadata, fresh slots are zeroed outside the graph."""
    case(Env(vefulix_folders, dtype, graphs=True), as_held("mix", dtype))


def test_hip_libraries_are_the_ones_running(env):
    CUTS.whole(env, as_held("one", env.dtype))
    assert ops.backend().name == "hip" and any("libme_core" in p for p in ops.loaded_libraries())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mix", "odd", "pages"])
def test_greedy_generation_through_the_scheduler(vefulix_folders, dtype, name):
    name = as_held(name, dtype)
    CUTS.greedy_through_the_engine(DEV, dtype, name, vefulix_folders(name), exact=dtype == "float32")


@pytest.mark.parametrize("name", ["mix", "mid", "flat", "pages"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_program_on_this_design(vefulix_folders, tmp_path, dtype, name):
    """bin/trace_run picks the model class by the folder's config: four live requests, portions beside single tokens, state
    slots and pages used again; also on models that keep only states or only pages."""
    name = as_held(name, dtype)
    folder = vefulix_folders(name)
    V = C.CONFIGS[name]["vocab"]
    lens = {"a": 100, "b": 64, "c": 30, "d": 77, "e": 50}
    ids = {r: helpers.random_ids(n, V, 900 + i) for i, (r, n) in enumerate(lens.items())}
    schedule = helpers.cuts_schedule({r: lens[r] for r in ("a", "b", "c", "d")}, [19, 1, 1, 2, 33, 1, 7, 1])
    steps = TR.steps_from_schedule(ids, schedule)
    last_c = max(i for i, st in enumerate(schedule) if "c" in st)
    for j, st in enumerate(helpers.cuts_schedule({"e": lens["e"]}, [5, 1, 40, 1])):
        a, b = st["e"]
        entry = {"id": "e", "tokens": ids["e"][a:b], "want": list(range(b - a))}
        i = last_c + 1 + j
        if i < len(steps):
            steps[i]["entries"].append(entry)
            if b == lens["e"]:
                steps[i]["end"].append("e")
        else:
            steps.append({"step": i, "entries": [entry], "end": ["e"] if b == lens["e"] else []})
    out = str(tmp_path / "o")
    TR.replay(folder, dtype, steps, out, max_tokens=TR.most_live_tokens(steps), page=C.PAGE[name])
    for r, g in TR.collect(steps, out, V).items():
        err = helpers.rel_err(g, C.plain_logits(folder, ids[r]))
        assert err <= TOL[getattr(torch, dtype)], f"{dtype} request {r}: {err:.3g}"


def test_offline_workload_row_with_random_weights(tmp_path, capsys):
    """The offline workload through the command line, on this design at a tiny size with random weights."""
    import json
    from mini_engine_amd import cli
    rc = cli.main(["--random-weights", "vefulix:tinyA", "--num-seqs", "6", "--max-prompt", "40", "--max-output", "8",
                   "--max-model-len", "64", "--max-num-seqs", "4", "--budget", "32", "--tokens-out", "-",
                   "--out", str(tmp_path / "bench.jsonl")])
    assert rc == 0
    lines = capsys.readouterr().out.strip().splitlines()
    row = json.loads(lines[-1])
    tokens = [json.loads(line) for line in lines[-7:-1]]
    assert [len(t) for t in tokens] == [8] * 6 and all(0 <= t < 256 for ts in tokens for t in ts)
    assert row["num_seqs"] == 6 and row["output_tokens"] == 48 and row["throughput_tok_s"] > 0
