"""The engine against a plain evaluation of whole sequences under every way of cutting the work, for any design.

`Cuts(configs, pages, plain_logits)`: the test configurations by name (dictionaries with "vocab"), their page sizes, and a
function (folder, token ids) -> float64 logits of every position. Each case takes `env` with .device, .dtype, .tol (optionally
.mean_tol: what the rows' errors have to stay within in the mean) and
.runner(name, pages, slots) -> (runner, manager, folder); the same cases run on the CPU (plain kernel twins, float32) and on
the GPU (HIP kernels, float32 and bfloat16). Pools start filled with NaN, so a read of a key or state nobody wrote poisons
the logits.
"""
from __future__ import annotations

import helpers
from helpers import Driver, random_ids, rel_err


def free_pages(manager) -> int:
    return min((manager.num_free_pages(g) for g in range(manager.num_groups)), default=1 << 30)


class Cuts:
    def __init__(self, configs: dict, pages: dict, plain_logits):
        self.configs, self.pages, self.plain_logits = configs, pages, plain_logits
        self.ALL = [self.whole, self.token_by_token, self.portions, self.batch_against_alone, self.long_decode, self.slots_start_from_zero]

    def vocab(self, name):
        return self.configs[name]["vocab"]

    def check(self, env, folder, ids, got, what):
        ref = self.plain_logits(folder, ids)[: got.shape[0]]
        err = rel_err(got, ref)
        assert err <= env.tol, f"{what}: error {err:.3g} > {env.tol:g}; first bad position {helpers.first_bad_row(got, ref, env.tol)}"
        mean = float(((got.double() - ref).abs().amax(-1) / ref.abs().max()).mean())
        assert got.shape[0] < 9 or mean <= getattr(env, "mean_tol", env.tol), f"{what}: mean error of the rows {mean:.3g} > {env.mean_tol:g}"

    def whole(self, env, name):
        """Each request alone and whole: one token, two, lengths around pages and chunks."""
        page = self.pages[name]
        for n in (1, 2, page, page + 1, 21, 50, 83):
            runner, manager, folder = env.runner(name, -(-n // page), 1)
            ids = random_ids(n, self.vocab(name), 100 + n)
            d = Driver(runner, manager)
            d.step({"r": ids}, end=["r"])
            self.check(env, folder, ids, d.result("r"), f"{name} whole n={n}")

    def token_by_token(self, env, name):
        """A whole request decoded one token at a time from its first token, beside the same request in one step."""
        page = self.pages[name]
        n = 45
        ids = random_ids(n, self.vocab(name), 200)
        runner, manager, folder = env.runner(name, 2 * -(-n // page), 2)
        d = Driver(runner, manager)
        for t in range(n):
            d.step({"r": ids[t:t + 1]})
        d.step({"w": ids})
        self.check(env, folder, ids, d.result("r"), f"{name} token by token")
        self.check(env, folder, ids, d.result("w"), f"{name} whole beside it")

    def portions(self, env, name):
        """Portions of changing size, down to two tokens and one, cut inside pages and chunks."""
        page = self.pages[name]
        n = 90
        ids = random_ids(n, self.vocab(name), 300)
        for pattern in ([2, 3, 5, 8, 13, 21, 2, 2], [17, 2, 1, 1, 2, 31, 2], [page, 2, page + 1, page - 1], [2]):
            runner, manager, folder = env.runner(name, -(-n // page), 1)
            d = Driver(runner, manager)
            pos, i = 0, 0
            while pos < n:
                c = min(pattern[i % len(pattern)], n - pos)
                d.step({"r": ids[pos:pos + c]})
                pos += c; i += 1
            self.check(env, folder, ids, d.result("r"), f"{name} portions {pattern}")

    def batch_against_alone(self, env, name):
        """Unequal requests in one batch, portions beside single tokens, against the plain evaluation of each alone; pages
        and state slots of ended requests are taken by later ones while others are live."""
        page, V = self.pages[name], self.vocab(name)
        lens = {"a": 40, "b": 23, "c": 9, "d": 61, "e": 30, "f": 1, "g": 17}
        ids = {r: random_ids(n, V, 400 + i) for i, (r, n) in enumerate(lens.items())}
        need = lambda r: -(-lens[r] // page)
        runner, manager, folder = env.runner(name, need("a") + need("d") + need("e"), 3)
        d = Driver(runner, manager)
        waiting, live, pos = list(lens), [], {}
        patterns = {"a": [11, 2, 9], "b": [23], "c": [2, 2, 5], "d": [7, 16, 3, 20], "e": [30], "f": [1], "g": [5, 12]}
        step_no = 0
        slots = len(manager.free_slots)
        while waiting or live:
            while waiting and len(live) < 3 and free_pages(manager) >= need(waiting[0]) and (slots == 0 or len(manager.free_slots) > 0):
                r = waiting.pop(0)
                live.append(r); pos[r] = 0
                manager.allocate(r, 0, 0)          # takes its state slot now, pages as it goes
            parts, ended = {}, []
            for r in live:
                plan, acc, take = patterns[r], 0, 1
                for c in plan:
                    if acc == pos[r]:
                        take = c
                        break
                    acc += c
                take = min(take, lens[r] - pos[r])
                if (step_no + len(r)) % 5 == 4 and pos[r] > 0:
                    continue                          # a request may sit a step out
                parts[r] = ids[r][pos[r]:pos[r] + take]
                pos[r] += take
                if pos[r] == lens[r]:
                    ended.append(r)
            step_no += 1
            if parts:
                d.step(parts, end=ended)
                for r in ended:
                    live.remove(r)
        for r in lens:
            self.check(env, folder, ids[r], d.result(r), f"{name} request {r} in the batch")
        assert len(manager.free_slots) == slots

    def long_decode(self, env, name):
        """A short prompt, then many single tokens over many page borders."""
        page = self.pages[name]
        n = 140
        ids = random_ids(n, self.vocab(name), 500)
        runner, manager, folder = env.runner(name, -(-n // page), 1)
        d = Driver(runner, manager)
        d.step({"r": ids[:6]})
        for t in range(6, n):
            d.step({"r": ids[t:t + 1]})
        self.check(env, folder, ids, d.result("r"), f"{name} long decode")

    def slots_start_from_zero(self, env, name):
        """A request that takes over the state slot and the pages of one that has ended starts from nothing."""
        page, V = self.pages[name], self.vocab(name)
        runner, manager, folder = env.runner(name, 4, 1)
        d = Driver(runner, manager)
        for i, n in enumerate((4 * page, 3, 2 * page + 1, 1)):
            ids = random_ids(n, V, 700 + i)
            d.step({f"r{i}": ids[:n // 2 + 1]})
            if n // 2 + 1 < n:
                d.step({f"r{i}": ids[n // 2 + 1:]}, end=[f"r{i}"])
            else:
                manager.free(f"r{i}")
            self.check(env, folder, ids, d.result(f"r{i}"), f"{name} request {i} in a used slot")

    def long_prompt(self, env, name, n=330, cuts=(147, 1, 1, 2, 3, 64, 65, 1)):
        """Keys and states hundreds of positions back: a prompt whole, and the same in portions whose last tokens are decoded
        alone, with a second request between them in the batch."""
        page = self.pages[name]
        ids, other = random_ids(n, self.vocab(name), 600), random_ids(40, self.vocab(name), 601)
        runner, manager, folder = env.runner(name, 2 * -(-n // page) + -(-40 // page), 3)
        d = Driver(runner, manager)
        d.step({"w": ids})
        pos, fed = 0, 0
        for c in cuts + (n - sum(cuts) - 8,) + (1,) * 8:
            step = {"r": ids[pos:pos + c]}
            pos += c
            if fed < 40:
                step["o"] = other[fed:fed + 4]
                fed += 4
            d.step(step)
        self.check(env, folder, ids, d.result("w"), f"{name} whole")
        self.check(env, folder, ids, d.result("r"), f"{name} cut")
        self.check(env, folder, other[:fed], d.result("o"), f"{name} beside it")

    def greedy_through_the_engine(self, device, dtype_name, name, folder, exact: bool):
        """Greedy generation through `LLM.generate`: the scheduler admits under a token budget, cuts prompts, batches
        portions beside decoding requests, takes and gives back pages and state slots; decode steps go through the
        fixed layouts (captured as graphs on a GPU) and run one ahead."""
        from mini_engine_amd import LLM, SamplingParams
        V = self.vocab(name)
        prompts = [random_ids(n, V, 800 + n) for n in (30, 12, 9, 1, 21)]
        llm = LLM(folder, dtype=dtype_name, device=device, kvcache_block_size=self.pages[name], num_kvcache_blocks=24, max_num_seqs=3,
                  max_num_batched_tokens=16, max_model_len=64, poison_cache=True)
        slots = len(llm.manager.free_slots)
        outs = llm.generate(prompts, SamplingParams(temperature=0, max_tokens=12, ignore_eos=True), use_tqdm=False)
        assert llm.runner.graphs is not None and llm.runner.graphs.replays > 0, "no decode step went through the fixed-layout path"
        llm.manager.check_invariants()
        assert len(llm.manager.free_slots) == slots and free_pages(llm.manager) >= 24
        for p, o in zip(prompts, outs):
            seq = list(p)
            assert len(o["token_ids"]) == 12
            for tok in o["token_ids"]:
                z = self.plain_logits(folder, seq)[-1]
                best = int(z.argmax())
                close = not exact and float(z[best] - z[tok]) < 8e-2 * float(z.abs().max())
                assert tok == best or close, f"{name} {dtype_name}: generated {tok}, the plain evaluation gives {best}"
                seq.append(tok)
