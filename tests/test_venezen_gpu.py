"""Venezen on the GPU: each new kernel form (slopes and sinks inside the attention kernels, values that are the keys, identity
experts, clamped gates, biases) against its plain twin at sizes of its own, then every layer, the engine's cuts, batches, page
reuse and long decoding in float32 and bfloat16 against the plain evaluation, windows at their edges, real layer sizes, decode steps
replayed as graphs, greedy generation through the scheduler, and the trace program on folders of this design."""
import pytest
import torch

import helpers
import kernel_twins as twin
import test_trace_run as TR
import venezen_cases as C
from mini_engine_amd.cache.manager import CacheManager
from mini_engine_amd.engine.runner import ModelRunner
from mini_engine_amd.kernels import ops
from mini_engine_amd.weights.loader import load_model
from test_venezen_cpu import edge_folder

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


def _wide(t):
    return t.cpu().float() if torch.is_tensor(t) and t.is_floating_point() else (t.cpu() if torch.is_tensor(t) else t)


# ------------------------------------------------------------------ attention: slopes, sinks, values that are the keys

def _batch(dtype, H, G, D, page, lens, news, seed):
    """Pages of keys (also the values), queries and metadata of requests that stand at `lens` tokens of which the last `news` are
    this step's; decode requests first. Pages that hold no visible key are not in the table."""
    torch.manual_seed(seed)
    B, MB = len(lens), max(-(-n // page) for n in lens)
    bt = torch.randperm(B * MB).view(B, MB).to(torch.int32).to(DEV)
    k = torch.randn(B * MB + 1, G, page, D, device=DEV).to(dtype)
    v = k.transpose(2, 3).contiguous()
    T = sum(news)
    q = (torch.randn(T, H * D, device=DEV) * 1.5).to(dtype)
    pos = torch.cat([torch.arange(n - m, n) for n, m in zip(lens, news)]).to(torch.int32).to(DEV)
    seq = torch.repeat_interleave(torch.arange(B), torch.tensor(news)).to(torch.int32).to(DEV)
    dn = sum(1 for m in news if m == 1)
    ctx = torch.tensor(lens, dtype=torch.int32, device=DEV)
    cu = torch.tensor([0] + list(torch.tensor(news[dn:]).cumsum(0)), dtype=torch.int32, device=DEV) if dn < B else None
    return q, k, v, bt, ctx, seq, pos, cu, dn, max(lens[:dn], default=0), max(lens[dn:], default=0)


@pytest.mark.parametrize("window", [None, 1, 2, 33, 200])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,page", [(4, 2, 128, 16), (5, 5, 32, 8), (6, 2, 48, 16), (1, 1, 128, 32), (24, 1, 32, 16), (3, 1, 16, 8), (8, 8, 128, 8), (4, 4, 20, 4)])
def test_attention_with_slopes_and_sinks(dtype, H, G, D, page, window):
    """Prompts, portions and single tokens in one batch, through every path: the matrix-core kernels for decoding and prompts, single
    tokens as prompts, the exact kernel; pages behind the window of the oldest query are given back (a table entry of -1)."""
    lens, news = [300, 41, 1, 700, 18, 130], [1, 1, 1, 90, 18, 128]
    q, k, v, bt, ctx, seq, pos, cu, dn, mdc, mpc = _batch(dtype, H, G, D, page, lens, news, D + H)
    if window:
        for b, (n, m) in enumerate(zip(lens, news)):
            first = max(0, n - m - window + 1) // page
            bt[b, :first] = -1
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], device=DEV)
    sinks = torch.linspace(-2.0, 4.0, H, device=DEV)
    run = lambda B, cast, **kw: B.paged_attention(*[cast(t) for t in (q, k, v, page, bt, ctx, seq, pos, cu)], dn, mdc, D ** -0.5, window, H, G, D,
                                                  max_prefill_context=mpc, **kw)
    tol = 1.5e-2 if dtype == torch.bfloat16 else 2e-5
    for s, z in ((slopes, sinks), (slopes, torch.zeros(H, device=DEV)), (slopes, None), (None, sinks)):
        want = run(twin, _wide, slopes=_wide(s), sinks=_wide(z))
        for forced in ({}, {"decode_as_prefill": True}, {"force_simple": True}):
            close(run(hip(), lambda t: t, slopes=s, sinks=z, **forced), want, tol)


@pytest.mark.parametrize("D,H,G", [(128, 4, 2), (64, 8, 8), (256, 4, 1)])
@pytest.mark.parametrize("window", [None, 3000])
def test_attention_with_slopes_over_cut_key_ranges(D, H, G, window):
    """Long contexts: partitions of a decode step and segments of a portion's key range, each with the distances from its own keys, and
    the sink joined where they meet; one far key stands out for a head with a small slope."""
    page = 16
    lens, news = [5000, 2100, 4500], [1, 1, 200]
    q, k, v, bt, ctx, seq, pos, cu, dn, mdc, mpc = _batch(torch.bfloat16, H, G, D, page, lens, news, D)
    far = 2100                                     # the last query of the portion, last head, asks for the key of position 2,100
    k[bt[2, far // page], G - 1, far % page] = (q[-1, -D:].float() * 12.0 * D ** -0.5).to(k.dtype)
    v = k.transpose(2, 3).contiguous()
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], device=DEV)
    slopes[-1] = 2.0 ** -12
    sinks = torch.linspace(0.0, 5.0, H, device=DEV)
    run = lambda B, cast, **kw: B.paged_attention(*[cast(t) for t in (q, k, v, page, bt, ctx, seq, pos, cu)], dn, mdc, D ** -0.5, window, H, G, D,
                                                  max_prefill_context=mpc, **kw)
    want = run(twin, _wide, slopes=slopes.cpu(), sinks=sinks.cpu())
    got = run(hip(), lambda t: t, slopes=slopes, sinks=sinks)
    close(got, want, 1.5e-2)
    without = run(twin, _wide, slopes=torch.zeros(H), sinks=sinks.cpu())
    assert float((without - want).abs().max()) > 0.05 * float(want.abs().max())
    k[bt[2, far // page], G - 1, far % page] = 0
    moved = run(hip(), lambda t: t, slopes=slopes, sinks=sinks)[-1, -D:].float() - got[-1, -D:].float()
    assert float(moved.abs().max()) > 0.1 * float(got.float().abs().max()), "the far key hardly shows"


@pytest.mark.parametrize("window", [None, 40])
@pytest.mark.parametrize("H,G,D,page", [(4, 2, 128, 16), (6, 3, 48, 8), (3, 3, 32, 16), (16, 1, 64, 16), (5, 5, 16, 8)])
@pytest.mark.parametrize("normed", [False, True])
def test_fused_decode_step_with_values_that_are_keys(H, G, D, page, window, normed):
    """One launch against the separate kernels bit for bit (attention aside) and against the twin; norm and rotation move the keys,
    not the values."""
    torch.manual_seed(D + H)
    lens = [300, 1, 41, 77, 16]
    B, MB = len(lens), max(-(-n // page) for n in lens)
    bt = torch.randperm(B * MB).view(B, MB).to(torch.int32).to(DEV)
    k = torch.randn(B * MB + 1, G, page, D, device=DEV).to(torch.bfloat16)
    v = torch.randn(B * MB + 1, G, D, page, device=DEV).to(torch.bfloat16)
    rows = torch.randn(B, (H + G) * D, device=DEV).to(torch.bfloat16)
    ctx = torch.tensor(lens, dtype=torch.int32, device=DEV)
    w = (torch.rand(D, device=DEV) + 0.5, torch.rand(D, device=DEV) + 0.5) if normed else (None, None)
    table = torch.randn(512, D // 2, 2, device=DEV) if normed else None
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], device=DEV)
    sinks = torch.zeros(H, device=DEV)
    kw = dict(sinks=sinks, slopes=slopes, values_are_keys=True)
    k1, v1, k2, v2 = k.clone(), v.clone(), k.clone(), v.clone()
    got = hip().decode_step_attention(rows.clone(), *w, 1e-5, table, k1, v1, page, bt, ctx, max(lens), D ** -0.5, window, H, G, D, **kw)
    pos = (ctx - 1).to(torch.int32)
    slots = (bt[torch.arange(B, device=DEV), (pos // page).long()] * page + pos % page).to(torch.int32)
    r = rows.clone()
    hip().qk_norm_rope_store(r, *w, 1e-5, table, pos, slots, k2, v2, H, G, D, page, values_are_keys=True)
    assert torch.equal(k1, k2) and torch.equal(v1, v2)
    seq = torch.arange(B, dtype=torch.int32, device=DEV)
    close(hip().paged_attention(r[:, :H * D], k2, v2, page, bt, ctx, seq, pos, None, B, max(lens), D ** -0.5, window, H, G, D, sinks=sinks, slopes=slopes), got, 1e-2)
    wide = {n: _wide(t) for n, t in kw.items()}
    want = twin.decode_step_attention(rows.cpu(), _wide(w[0]), _wide(w[1]), 1e-5, _wide(table), k.cpu(), v.cpu(), page, bt.cpu(), ctx.cpu(), max(lens),
                                      D ** -0.5, window, H, G, D, **wide)
    close(got, want, 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,G,D,page", [(300, 4, 2, 128, 16), (40, 4, 2, 64, 16), (9, 3, 3, 48, 8), (150, 6, 2, 32, 8), (1, 5, 1, 80, 32), (130, 2, 2, 20, 4)])
def test_store_of_keys_that_are_values(dtype, T, H, G, D, page):
    """Every form of the kernel (tiles of tokens, vectors, pairs), with and without norm and rotation, rows inside wider ones, skipped
    slots, runs of slots that begin anywhere."""
    torch.manual_seed(T + D)
    pages = -(-T // page) + 3
    slots = torch.arange(5, 5 + T, dtype=torch.int32, device=DEV)
    slots[T // 2:] = torch.randperm(T - T // 2, device=DEV).to(torch.int32) + 5 + T // 2
    if T > 4:
        slots[3] = -1
    pos = torch.randint(0, 64, (T,), device=DEV, dtype=torch.int32)
    for w, table in (((None, None), None), ((torch.rand(D, device=DEV), torch.rand(D, device=DEV)), torch.randn(64, D // 2, 2, device=DEV))):
        wide = torch.randn(T, (H + G) * D + 16, device=DEV).to(dtype)
        mine, theirs = wide[:, : (H + G) * D], wide.cpu()[:, : (H + G) * D].clone()
        raw = mine[:, H * D:].clone()
        kc, vc = torch.zeros(pages, G, page, D, device=DEV, dtype=dtype), torch.zeros(pages, G, D, page, device=DEV, dtype=dtype)
        kc2, vc2 = kc.cpu().clone(), vc.cpu().clone()
        hip().qk_norm_rope_store(mine, *w, 1e-5, table, pos, slots, kc, vc, H, G, D, page, values_are_keys=True)
        twin.qk_norm_rope_store(theirs, *[_wide(t) for t in w], 1e-5, _wide(table), pos.cpu(), slots.cpu(), kc2, vc2, H, G, D, page, values_are_keys=True)
        assert torch.equal(vc.cpu(), vc2) and torch.equal(mine[:, H * D:], raw)
        close(kc, kc2, 1e-2 if dtype == torch.bfloat16 else 1e-5)
        close(mine[:, : H * D], theirs[:, : H * D], 1e-2 if dtype == torch.bfloat16 else 1e-5)


def test_exact_attention_of_heads_beyond_512_dimensions():
    """A latent of 600 with a rotating part: what no matrix-core kernel takes."""
    q, k, v, bt, ctx, seq, pos, cu, dn, mdc, mpc = _batch(torch.bfloat16, 3, 1, 640, 16, [70, 20], [1, 20], 9)
    args = lambda cast: [cast(t) for t in (q, k, v, 16, bt, ctx, seq, pos, cu)] + [dn, mdc, 0.05, None, 3, 1, 640]
    close(hip().paged_attention(*args(lambda t: t)), twin.paged_attention(*args(_wide)), 1e-2)


# ------------------------------------------------------------------ experts, biases, sums

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n,F,E,Z,top", [(5, 40, 24, 6, 2, 3), (300, 64, 40, 8, 4, 3), (1500, 128, 72, 4, 4, 2), (70, 36, 20, 5, 3, 8), (3, 64, 16, 1, 63, 4),
                                           (64, 96, 48, 12, 1, 1), (900, 264, 136, 2, 1, 3), (17, 50, 9, 3, 0, 2)])
def test_experts_with_a_clamped_gate_and_identity_experts(dtype, T, n, F, E, Z, top):
    """Every form of the kernels (tiles of 16, 64 and 128 rows, one wave per output, the choice inside the sort) against the twin;
    limits that bite on gates from above only and on ups at both sides; rows inside wider ones."""
    torch.manual_seed(T + F)
    wide = torch.randn(T, n + 8, device=DEV).to(dtype)
    x = wide[:, :n]
    router = torch.randn(E + Z, n, device=DEV) * n ** -0.5
    rule = ops.RouteRule("softmax", correction=torch.randn(E + Z, device=DEV) * 0.1, normalise=True, scale=1.7)
    gu = (torch.randn(E, 2 * F, n, device=DEV) * 2 * n ** -0.5).to(dtype)
    down = (torch.randn(E, n, F, device=DEV) * F ** -0.5).to(dtype)
    ids, weights = hip().moe_route(x, router, top, 1, 1, rule)
    assert Z == 0 or bool((ids >= E).any())
    tol = 2e-2 if dtype == torch.bfloat16 else 2e-5
    for clamp in ((0.7, 1.702), (100.0, 1.0), None):
        want = twin.routed_experts(x.cpu(), ids.cpu(), weights.cpu(), gu.cpu(), down.cpu(), clamp=clamp, routed=E + Z)
        close(hip().route_and_run_experts(x, router, top, 1, 1, gu, down, rule=rule, clamp=clamp), want, tol)
        for forced in ({}, {"force_simple": True}, {"tile_rows": 16}, {"tile_rows": 64}, {"tile_rows": 128}):
            got = hip().routed_experts(x, ids, weights, gu, down, clamp=clamp, routed=E + Z, **forced)
            close(got, want, tol)
            if Z:                                # an identity expert's part is exact
                t, j = (ids >= E).nonzero()[0].tolist()
                assert torch.allclose(got[j, t], x[t].float() * weights[t, j], rtol=1e-6)
    if Z:                                        # every pair an identity one: no expert's weights are read
        some = torch.full_like(ids, E) + torch.arange(top, device=DEV, dtype=torch.int32)[None, :] % Z
        got = hip().routed_experts(x, some, weights, torch.full_like(gu, float("nan")), torch.full_like(down, float("nan")), routed=E + Z)
        assert torch.allclose(got, x.float()[None] * weights.t()[:, :, None], rtol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,F", [(1, 256), (37, 24), (5, 13), (700, 100), (64, 3072), (9000, 40), (20, 6000)])
def test_silu_and_mul_with_biases(dtype, T, F):
    torch.manual_seed(T + F)
    gu, bias = torch.randn(T, 2 * F, device=DEV).to(dtype), torch.randn(2 * F, device=DEV)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    wide = torch.randn(T, 2 * F + 24, device=DEV).to(dtype)
    for at in (8, 3):                              # rows inside wider ones, at whole pieces and not
        close(hip().glu_clamped(wide[:, at:at + 2 * F], 0.8, 1.3), twin.glu_clamped(wide.cpu()[:, at:at + 2 * F], 0.8, 1.3), tol)
    close(hip().silu_and_mul(gu, bias=bias), twin.silu_and_mul(gu.cpu(), bias.cpu()), tol)
    close(hip().silu_and_mul(gu), twin.silu_and_mul(gu.cpu()), tol)


@pytest.mark.parametrize("M,F,K", [(1, 1536, 1024), (8, 3072, 1024), (16, 96, 40), (3, 12, 136), (24, 512, 1024), (40, 3072, 1024), (200, 512, 256), (128, 1536, 1024)])
def test_gate_and_up_with_biases_or_a_clamp_in_the_products_epilogue(M, F, K):
    """Both products that gate in their epilogue, against the twin, and against the product with the activation behind it."""
    torch.manual_seed(M + F)
    x, w = torch.randn(M, K, device=DEV).to(torch.bfloat16), (torch.randn(2 * F, K, device=DEV) * K ** -0.5).to(torch.bfloat16)
    bias = torch.randn(2 * F, device=DEV)
    assert ops.gated_linear_fuses(x, w)
    for kw in ({"bias": bias}, {"clamp": (0.6, 1.702)}, {"clamp": (50.0, 0.7)}, {}):
        want = twin.gated_linear(x.cpu(), w.cpu(), **{n: _wide(t) for n, t in kw.items()})
        close(hip().gated_linear(x, w, **kw), want, 1e-2)
    gu = hip().linear(x, w)
    close(hip().gated_linear(x, w, bias=bias), hip().silu_and_mul(gu, bias=bias), 3e-2)
    close(hip().gated_linear(x, w, clamp=(0.6, 1.702)), hip().glu_clamped(gu, 0.6, 1.702), 3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n", [(5, 64), (37, 50), (600, 132), (1, 3)])
def test_sums_with_a_bias_in_front_of_a_norm_without_one(dtype, T, n):
    torch.manual_seed(T + n)
    f = lambda *s: torch.randn(*s, device=DEV)
    x, a, b, bias, w = f(T, 1, n), f(3, T, n), f(T, n).to(dtype), f(n), f(n)
    rows = torch.randint(0, T, (7,), device=DEV, dtype=torch.int32)
    for terms, norm, pick in (([a, b], (w, None, 1e-5, True), None), ([b], (w, None, 1e-5, False), rows), ([a], None, None), ([], (w, None, 1e-5, True), None)):
        got_new, got = hip().stream_mix_norm(x, 1, terms, None, None, None, norm, dtype, rows=pick, bias=bias)
        want_new, want = twin.stream_mix_norm(x.cpu(), 1, [t.cpu() for t in terms], None, None, None, None if norm is None else (w.cpu(),) + norm[1:], dtype,
                                              rows=None if pick is None else pick.cpu(), bias=bias.cpu())
        close(got_new, want_new, 2e-6)
        close(got, want, 1e-2 if dtype == torch.bfloat16 else 1e-5)


# ------------------------------------------------------------------ the engine against the plain evaluation

def as_held(name, dtype):
    """The configuration that a dtype is held to the tolerance on, row by row: in bfloat16 the one whose tokens take every expert (a
    choice between two close scores may fall otherwise there; what is chosen is held by the experts' own test and in the mean)."""
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
        manager = CacheManager(pages, C.PAGE[name], ModelRunner.windows_of(model), num_state_slots=0, enable_prefix_caching=False)
        options = dict(use_graphs=True, mixed_graphs_after=1) if self.graphs else {}
        return ModelRunner(model, manager, self.dtype, self.device, 1024, poison_cache=True, **options), manager, folder


@pytest.fixture(scope="module")
def venezen_folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = C.make_folder(name, str(tmp_path_factory.mktemp(f"venezen_{name}")))
        return made[name]

    return get


@pytest.fixture(scope="module", params=DTYPES, ids=["float32", "bfloat16"])
def env(request, venezen_folders):
    return Env(venezen_folders, request.param)


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


@pytest.mark.parametrize("dtype", DTYPES, ids=["float32", "bfloat16"])
@pytest.mark.parametrize("size", [1, 2, 8, 9, 40])
def test_window_edges(tmp_path_factory, size, dtype):
    C.window_edges(Env(edge_folder(tmp_path_factory, size), dtype), f"edge{size}", 0)


def test_real_layer_sizes(venezen_folders):
    C.real_sizes(Env(venezen_folders, torch.float32), Env(venezen_folders, torch.bfloat16))


def test_real_layer_sizes_with_a_choice_of_experts(venezen_folders):
    C.real_sizes(Env(venezen_folders, torch.float32), Env(venezen_folders, torch.bfloat16), "routed", every_row=False)


@pytest.mark.parametrize("dtype", DTYPES, ids=["float32", "bfloat16"])
@pytest.mark.parametrize("case", [CUTS.token_by_token, CUTS.long_decode, CUTS.batch_against_alone], ids=lambda c: c.__name__)
def test_cuts_through_captured_steps(venezen_folders, case, dtype):
    """The same with decode steps (and small steps that come up again) replayed as graphs."""
    case(Env(venezen_folders, dtype, graphs=True), as_held("mix", dtype))


def test_hip_libraries_are_the_ones_running(env):
    CUTS.whole(env, as_held("one", env.dtype))
    assert ops.backend().name == "hip" and any("libme_core" in p for p in ops.loaded_libraries())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mix", "odd", "windows"])
def test_greedy_generation_through_the_scheduler(venezen_folders, dtype, name):
    name = as_held(name, dtype)
    CUTS.greedy_through_the_engine(DEV, dtype, name, venezen_folders(name), exact=dtype == "float32")


@pytest.mark.parametrize("name", ["mix", "mid", "windows", "pages"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_program_on_this_design(venezen_folders, tmp_path, dtype, name):
    """bin/trace_run picks the model class by the folder's config: four live requests, portions beside single tokens, pages used again;
    also on models whose layers are all windowed or all unbounded."""
    name = as_held(name, dtype)
    folder = venezen_folders(name)
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
    rc = cli.main(["--random-weights", "venezen:tinyA", "--num-seqs", "6", "--max-prompt", "40", "--max-output", "8",
                   "--max-model-len", "64", "--max-num-seqs", "4", "--budget", "32", "--tokens-out", "-",
                   "--out", str(tmp_path / "bench.jsonl")])
    assert rc == 0
    lines = capsys.readouterr().out.strip().splitlines()
    row = json.loads(lines[-1])
    tokens = [json.loads(line) for line in lines[-7:-1]]
    assert [len(t) for t in tokens] == [8] * 6 and all(0 <= t < 256 for ts in tokens for t in ts)
    assert row["num_seqs"] == 6 and row["output_tokens"] == 48 and row["throughput_tok_s"] > 0
