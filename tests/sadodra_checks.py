"""Checks of the Sadodra mechanisms and engine schedules against the float64 oracle, written once for
both backends: ``Env("torch", "cpu", ...)`` runs the PyTorch reference ops, ``Env("hip", "cuda", ...)``
the HIP kernels.  Every mixer is driven alone, over shuffled pages, whole and in portions, with an
input of the test's making."""
import numpy as np
import torch

import sadodra_cases as C
import sadodra_oracle as O
from byzantine_consensus_llm_agents_amd.models.config import SadodraConfig
from byzantine_consensus_llm_agents_amd.models.sadodra import SadodraModel
from byzantine_consensus_llm_agents_amd.ops import get_ops


class Env:
    def __init__(self, backend, device, dtype=torch.float32):
        self.backend, self.device, self.dtype = backend, device, dtype
        self.ops = get_ops(backend)
        self.noise = 0.0   # bf16: the worst row error that rounding alone causes in this case (`measure_noise`)

    def measure_noise(self, path, cfg, sd, n=150):
        """Run the reference ops in this dtype over two prompts: what rounding alone does to the worst row."""
        if self.dtype == torch.float32:
            return
        n = min(n, cfg["max_positions"])
        ref = C.engine(path, backend="torch", dtype=self.dtype, pool_tokens=max(256, n + 16), max_len=max(512, n))
        for seed in (77, 78):
            toks = C.tokens(n, cfg["vocab"], seed)
            got = ref.stream_step([("n", toks, list(range(n)))], end=["n"]).double().numpy()
            self.noise = max(self.noise, float(row_error(got, O.forward(sd, cfg, toks)).max()))
        ref.shutdown()

    def close(self, got, want, tol=None, noise=0.0):
        """fp32: elementwise.  bf16: the row error relative to the spread of the expected values;
        ``noise`` is what rounding alone does to the worst row, measured on the reference ops in bf16."""
        got, want = got.detach().double().cpu().numpy(), np.asarray(want)
        assert got.shape == want.shape, (got.shape, want.shape)
        noise = max(noise, self.noise)
        if self.dtype == torch.float32:
            tol = tol or 3e-4
            np.testing.assert_allclose(got, want, atol=tol, rtol=tol)
        else:
            err = row_error(got, want)
            # (a softmax between two near equal keys turns a rounding into a large step of one row: a
            # few rows may lie further out than the worst of the sample)
            assert float(err.max()) < max(0.1, 4.0 * noise), (float(err.max()), noise)
            assert float(np.quantile(err, 0.95)) < max(0.06, 1.3 * noise), (float(np.quantile(err, 0.95)), noise)
            assert float(np.median(err)) < max(0.03, 0.7 * noise), (float(np.median(err)), noise)

    def t(self, x, dtype=None):
        return torch.as_tensor(np.asarray(x)).to(device=self.device, dtype=dtype or self.dtype, copy=True)


def row_error(got, want):
    return np.sqrt(((got - want) ** 2).mean(-1)) / max(float(want.std()), 1e-6)


def rand_bf16(g, *shape, scale=1.0):
    return (torch.randn(*shape, generator=g) * scale).to(torch.bfloat16).float()


# ------------------------------------------------------------------ embedding, norms, feed-forward
def check_embedding(env, W=44):
    g = torch.Generator().manual_seed(W)
    table, pos = rand_bf16(g, 11, W), rand_bf16(g, 9, W)
    toks, ps = [3, 0, 10, 3, 7], [0, 8, 2, 3, 1]
    i32 = dict(dtype=torch.int32, device=env.device)
    x, h = env.ops.embed_position(torch.tensor(toks, **i32), torch.tensor(ps, **i32), env.t(table), env.t(pos), env.dtype)
    want = table.double().numpy()[toks] + pos.double().numpy()[ps]
    assert x.dtype == torch.float32 and h.dtype == env.dtype
    np.testing.assert_allclose(x.double().cpu().numpy(), want, atol=1e-6)
    env.close(h, want, 1e-6)


def check_layer_norms(env, W=44, T=5):
    """x += layer_norm(y), its three followers (copy, layer norm, nothing), y typed and fp32; rows with a
    large mean show a norm that does not take it off."""
    g = torch.Generator().manual_seed(W)
    x0, y = rand_bf16(g, T, W), rand_bf16(g, T, W) + 3.0
    y = y.to(torch.bfloat16).float()
    w1, b1, w2, b2 = (rand_bf16(g, W) for _ in range(4))
    f = lambda a: env.t(a, torch.float32)  # noqa: E731
    d = lambda a: a.double().numpy()  # noqa: E731
    post, fin = ("ln", f(w1), f(b1), 1e-5), ("ln", f(w2), f(b2), 1e-3)
    want = d(x0) + O.layer_norm(d(y), d(w1), d(b1), 1e-5)
    x = f(x0)
    h = env.ops.residual_post_norm(x, env.t(y), post, ("copy",), env.dtype)
    np.testing.assert_allclose(x.double().cpu().numpy(), want, atol=2e-5)
    env.close(h, want, 2e-5)
    want = want + O.layer_norm(d(y) * 2, d(w1), d(b1), 1e-5)
    h = env.ops.residual_post_norm(x, f(y) * 2, post, fin, env.dtype)
    np.testing.assert_allclose(x.double().cpu().numpy(), want, atol=4e-5)
    env.close(h, O.layer_norm(want, d(w2), d(b2), 1e-3), 5e-5)
    assert env.ops.residual_post_norm(x, env.t(y), post, None, env.dtype) is None
    np.testing.assert_allclose(x.double().cpu().numpy(), want + O.layer_norm(d(y), d(w1), d(b1), 1e-5), atol=5e-5)


def check_feed_forward(env, W, ff, T=23):
    cfg, model, sd = _model(env, [C.A(ff)], W, seed=ff)
    for n in ("gate", "up"):
        sd[f"l0.mlp.{n}"] *= 3    # reach both tails of the activation
    model.load_hf_state_dict(sd)
    h = rand_bf16(torch.Generator().manual_seed(ff), T, W)
    env.close(model._feed_forward(model.layers[0], env.t(h)), O.feed_forward(O.to_f64(sd), "l0.mlp.", h.double().numpy()))


# ------------------------------------------------------------------ one mixer alone
def _model(env, layers, width, seed):
    cfg = SadodraConfig.from_dict(C.config(layers, width=width, vocab=29), "t")
    model = SadodraModel(cfg, env.ops, env.device, env.dtype)
    return cfg, model, model.random_state_dict(seed, std=0.2)


def oracle_mixer(layers, sd, hs, eps=1e-5):
    """What the LAST layer's mixer makes of its input (a lender's latents come from the lender's own)."""
    last = len(layers) - 1
    m, p = layers[last]["mixer"], f"l{last}.mix."
    if layers[last]["type"] == "attention":
        return O.attention(sd, p, m, hs[last], eps)
    src = m.get("kv_from", last)
    return O.latent_attention(sd, p, m, hs[last], O.latent(sd, f"l{src}.mix.", hs[src], eps))


def run_mixer(env, layers, T, cuts=None, craft=None, seed=0, width=40):
    """Drive the LAST layer's mixer alone over the portions ``cuts`` of one sequence (the layer whose
    latents it borrows runs too, from an input of its own).  ``craft(sd, hs)`` may edit the weights
    and the per-layer inputs.  Returns (got [T, W], want [T, W], float64 weights, float64 inputs)."""
    cfg, model, sd = _model(env, layers, width, seed)
    g = torch.Generator().manual_seed(seed + 100)
    hs = [rand_bf16(g, T, width) for _ in layers]
    if craft:
        craft(sd, hs)
    model.load_hf_state_dict(sd)
    sd64, hs64 = O.to_f64(sd), [h.double().numpy() for h in hs]
    want = oracle_mixer(layers, sd64, hs64)
    last = len(layers) - 1
    pages = C.Pages([T, 5, T], seed=seed, device=env.device)
    ks, vs = model.alloc_kv(pages.num_blocks, 16, env.dtype)
    for t in {id(t): t for t in ks + vs}.values():
        t.fill_(3.0)     # a freed page's stale content
    src = layers[last]["mixer"].get("kv_from", last)
    at, outs = 0, []
    for c in cuts or [T]:
        meta = pages.meta([(2, at, c)])
        for i in sorted({src, last}):
            m, L, h = model.cfg.layers[i].mixer, model.layers[i], env.t(hs[i][at:at + c])
            fn = model._attention if layers[i]["type"] == "attention" else model._latent_attention
            y = fn(m, L, h, meta, ks[i], vs[i], None)
        outs.append(y)
        at += c
    return torch.cat(outs), want, sd64, hs64


def loud_value(pos, factor):
    """Input row ``pos`` scaled up: its key is normed whatever the size, its value (the key before the
    norm) is ``factor`` times the others, so it dominates the output of every query that sees it."""
    def craft(sd, hs):
        for h in hs:
            h[pos] *= factor
    return craft


def check_window_edge(env, window=9, T=40, loud=10, cuts=None, seed=5):
    """Position loud + window - 1 is the last that sees the loud row, loud the first."""
    layers = [C.A(0, heads=2, kv_heads=1, dim=16, window=window, softcap=2.0, scale=0.05)]   # one head's slope is 2^-8: nearly flat
    got, want, _, _ = run_mixer(env, layers, T, cuts, loud_value(loud, max(100.0, 12.0 * window)), seed=seed)
    env.close(got, want, 1e-2)   # (the loud rows are hundreds of times larger)
    # rows that do not see it, on their own scale
    quiet = [t for t in range(T) if not loud <= t < loud + window]
    env.close(got[quiet], want[quiet])
    assert np.abs(want[loud + window - 1]).max() > 4 * np.abs(want[loud + window]).max()
    assert np.abs(want[loud]).max() > 4 * np.abs(want[loud - 1]).max()
    return got


def planted_pair(kind, i, j, gain, width):
    """Rows i and j of the input point opposite ways, all others are orthogonal to them, and the
    projections copy the input, the key's with that direction turned round: query i's score on key j
    stands far above the others, its own included."""
    def craft(sd, hs):
        p = "l0.mix."
        eye, turned = torch.eye(width), torch.eye(width)
        turned[0, 0] = -1.0
        sd[p + "q"] = (eye * gain).to(torch.bfloat16)
        if kind == "attention":
            sd[p + "k"] = turned.to(torch.bfloat16)
            sd[p + "q.norm"], sd[p + "k.norm"] = (torch.ones(width, dtype=torch.bfloat16) for _ in range(2))
        else:
            sd[p + "dkv"] = turned.to(torch.bfloat16)
            sd[p + "dkv.norm"] = torch.ones(width, dtype=torch.bfloat16)
            sd[p + "uk"] = eye.to(torch.bfloat16)
        for h in hs:
            h[:, 0] = 0.0
            h[i] = h[j] = 0.0
            h[i, 0], h[j, 0] = 2.0, -2.0
    return craft


def check_far_key(env, kind, T=300, i=290, j=3, cuts=None):
    """One key among hundreds carries a query's output; without it the output is another one."""
    W = 16
    if kind == "attention":   # one head: slope 2^-8, no window
        layers = [C.A(0, heads=1, kv_heads=1, dim=W, window=0, softcap=20.0, temp=(0.5, 64), scale=1.0)]
        gain = 1.0
    else:
        layers = [C.L(0, heads=1, dim=W, vdim=W, kv_rank=W, scale=1.0)]
        gain = 3.0
    got, want, sd, hs = run_mixer(env, layers, T, cuts, planted_pair(kind, i, j, gain, W), seed=6, width=W)
    env.close(got, want)
    cut = [h.copy() for h in hs]
    cut[0][j] = cut[0][j + 1]
    without = oracle_mixer(layers, sd, cut)
    assert np.abs(want[i] - without[i]).max() > 0.2 * np.abs(want[i]).max()
    assert np.abs(want[i + 1] - without[i + 1]).max() < 0.2 * np.abs(want[i + 1]).max()   # (only that query)


# ------------------------------------------------------------------ engine schedules
def whole_prompt(env, cfg, sd, eng, n=45):
    toks = C.tokens(n, cfg["vocab"], 1)
    env.close(eng.stream_step([("a", toks, list(range(n)))], end=["a"]), O.forward(sd, cfg, toks))


def stream_after_every_layer(env, cfg, sd, eng):
    toks = C.tokens(19, cfg["vocab"], 2)
    want = []
    O.forward(sd, cfg, toks, want)
    pages = C.Pages([19], device=env.device)
    k, v = eng.model.alloc_kv(pages.num_blocks, 16, env.dtype)
    got = []
    eng.model.forward(torch.tensor(toks, dtype=torch.int32, device=env.device), pages.meta([(0, 0, 19)]), k, v, trace=got)
    assert len(got) == len(want) == len(cfg["layers"])
    for a, b in zip(got, want):
        env.close(a, b)


def prefill_then_token_by_token(env, cfg, sd, eng, n=70, first=30):
    toks = C.tokens(n, cfg["vocab"], 3)
    want = O.forward(sd, cfg, toks)
    env.close(eng.stream_step([("d", toks[:first], [0, 1, first - 1])]), want[[0, 1, first - 1]])
    got = [eng.stream_step([("d", toks[p:p + 1], [0])], end=["d"] if p == n - 1 else []) for p in range(first, n)]
    env.close(torch.cat(got), want[first:])   # crosses page borders and every window's edge


def first_tokens_one_by_one(env, cfg, sd, eng):
    toks = C.tokens(7, cfg["vocab"], 4)
    want = O.forward(sd, cfg, toks)
    got = [eng.stream_step([("f", toks[p:p + 1], [0])], end=["f"] if p == 6 else []) for p in range(7)]
    env.close(torch.cat(got), want)


def portions(env, cfg, sd, eng, sizes):
    n = sum(sizes)
    toks = C.tokens(n, cfg["vocab"], 5)
    want = O.forward(sd, cfg, toks)
    at, got = 0, []
    for i, s in enumerate(sizes):
        got.append(eng.stream_step([("p", toks[at:at + s], list(range(s)))], end=["p"] if i == len(sizes) - 1 else []))
        at += s
    env.close(torch.cat(got), want)


def mixed_batches_and_reuse(env, cfg, sd, eng, lens=(70, 33, 18, 64, 41, 90, 5, 36)):
    """Up to four live requests, portions beside single tokens, rows sitting out; twice as many
    requests as rows over a pool smaller than the work: pages and rows are used again."""
    reqs = {f"r{i}": C.tokens(n, cfg["vocab"], 10 + i) for i, n in enumerate(lens)}
    want = {k: O.forward(sd, cfg, t) for k, t in reqs.items()}
    at = {k: 0 for k in reqs}
    waiting, live, step = list(reqs), [], 0
    free_at_start = eng.blocks.num_free_blocks
    got, expect = [], []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        entries, end = [], []
        for j, k in enumerate(live):
            if (step + j) % 5 == 4 and at[k] > 0:
                continue
            take = [1, 2, 16, 7, 1, 19][(step + j) % 6] if at[k] > 0 else [20, 3, 16][j % 3]
            take = min(take, len(reqs[k]) - at[k])
            entries.append((k, reqs[k][at[k]:at[k] + take], list(range(take))))
            expect.append(want[k][at[k]:at[k] + take])
            at[k] += take
            if at[k] == len(reqs[k]):
                end.append(k)
        if entries:
            got.append(eng.stream_step(entries, end))
        live = [k for k in live if k not in end]
        step += 1
    env.close(torch.cat(got), np.concatenate(expect))
    assert eng.blocks.num_free_blocks == free_at_start and not any(eng.slots)
    assert sum(lens) > 16 * free_at_start / 2


def follow_greedy(cfg, sd, prompt, out, tie=1e-3):
    """Every generated id is the oracle's greedy step on what came before (near ties end the walk)."""
    seq = list(prompt)
    for tok in out:
        logits = O.forward(sd, cfg, seq)[-1]
        top2 = np.sort(logits)[-2:]
        if float(top2[1] - top2[0]) < tie * max(1.0, float(logits.std())):
            return
        assert tok == int(logits.argmax())
        seq.append(tok)


def greedy_generation(env, cfg, sd, eng, tie=1e-3):
    prompts = [C.tokens(n, cfg["vocab"], 20 + n) for n in (9, 31, 16, 2, 40, 23)]
    budgets = (6, 4, 17, 5, 3, 11)
    outs = eng.generate_ids(prompts, max_tokens=list(budgets), temperature=0.0)
    for p, out, n in zip(prompts, outs, budgets):
        assert len(out) == n
        follow_greedy(cfg, sd, p, out, tie)


def shared_prefixes(env, cfg, sd, eng, tie=1e-3):
    """Prompts that share full pages with earlier ones skip them (prefix cache) and generate the same."""
    base = C.tokens(50, cfg["vocab"], 41)
    first = eng.generate_ids([base + [1, 2]], 4)[0]
    before = eng.stats["cached_tokens"]
    prompts = [base + [1, 2], base[:40] + [3], base + [5] * 9]
    outs = eng.generate_ids(prompts, 4)
    assert eng.stats["cached_tokens"] - before >= 48 + 32 + 48
    for p, out in zip(prompts + [base + [1, 2]], outs + [first]):
        follow_greedy(cfg, sd, p, out, tie)


def drawn_configuration(env, tmp_path, seed, pool_tokens=256, cfg=None):
    cfg = cfg or C.random_config(seed)
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=seed))
    a, b = C.tokens(60, cfg["vocab"], seed), C.tokens(23, cfg["vocab"], seed + 100)
    wa, wb = O.forward(sd, cfg, a), O.forward(sd, cfg, b)
    env.measure_noise(path, cfg, sd)
    eng = C.engine(path, backend=env.backend, dtype=env.dtype, pool_tokens=pool_tokens)
    try:
        env.close(eng.stream_step([("w", a, list(range(60)))], end=["w"]), wa)
        at, got, want = 0, [], []
        for i, s in enumerate([3, 2, 30, 1, 1, 17, 2, 4]):
            entries = [("a", a[at:at + s], list(range(s))), ("b", b[i:i + 1], [0])]
            want += [wa[at:at + s], wb[i:i + 1]]
            at += s
            got.append(eng.stream_step(entries))
        env.close(torch.cat(got), np.concatenate(want))
        assert at == 60
        eng.stream_step([("b", b[8:], [])], end=["a", "b"])
        assert not any(eng.slots)
    finally:
        eng.shutdown()
