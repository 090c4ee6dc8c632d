"""Sadodra on the HIP backend against the float64 oracle: every mechanism's kernels alone (fp32 and
bf16), the new HIP ops against their PyTorch fp32 references at larger shapes, packed steps of the
engine (prompt portions beside single tokens, page reuse, shared prefixes), and greedy generation
through the scheduler with captured decode graphs."""
import pytest
import torch

import sadodra_cases as C
import sadodra_checks as K
import sadodra_oracle as O
from byzantine_consensus_llm_agents_amd.ops import reference as ref
from test_sadodra_cpu import ATTENTION, LATENT
from test_seqmix_kernels_gpu import _paged

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
DEV = "cuda"


@pytest.fixture(params=DTYPES)
def env(request):
    e = K.Env("hip", "cuda", getattr(torch, request.param))
    assert e.ops.name == "hip"
    return e


def _tol(dtype):
    return dict(atol=2e-2, rtol=2e-2) if dtype == torch.bfloat16 else dict(atol=3e-5, rtol=3e-5)


# ------------------------------------------------------------------ mechanisms
def test_embedding_and_layer_norms(env):
    for W in (44, 33, 256, 1030, 1029, 2048, 5000, 12288, 16384, 9001):   # every register form, on and off the 4-column grid
        K.check_embedding(env, W)
        K.check_layer_norms(env, W)


@pytest.mark.parametrize("W,ff", [(40, 24), (33, 41), (64, 7), (128, 520)])
def test_feed_forward(env, W, ff):
    K.check_feed_forward(env, W, ff)


@pytest.mark.parametrize("name", list(ATTENTION))
def test_attention_whole_and_in_portions(env, name):
    for cuts in (None, [2, 14, 1, 1, 17, 2, 8]):
        got, want, _, _ = K.run_mixer(env, ATTENTION[name], 45, cuts, seed=3)
        env.close(got, want)


@pytest.mark.parametrize("name", list(LATENT))
def test_latent_attention_whole_and_in_portions(env, name):
    for cuts in (None, [2, 14, 1, 1, 17, 2, 8]):
        got, want, _, _ = K.run_mixer(env, LATENT[name], 45, cuts, seed=3)
        env.close(got, want)


@pytest.mark.parametrize("heads,kv,dim,window", [(4, 2, 32, 70), (8, 4, 128, 80), (3, 1, 48, 0), (17, 1, 16, 40), (2, 2, 64, 150),
                                                 (4, 4, 96, 130), (2, 1, 192, 64), (2, 2, 256, 0), (1, 1, 144, 33), (2, 1, 300, 20)])
def test_attention_exact_and_wide_heads(env, heads, kv, dim, window):
    """Heads on the 16-wide MFMA grid (the straight-line instances) and off it, GQA groups above the 16
    MFMA columns, windows longer than a decode split, several 64-row tiles."""
    layers = [C.A(0, heads=heads, kv_heads=kv, dim=dim, window=window, softcap=12.0, temp=(0.4, 50), scale=0.2)]
    got, want, _, _ = K.run_mixer(env, layers, 200, [150, 1, 1, 40] + [1] * 8, seed=heads, width=48)
    env.close(got, want)


@pytest.mark.parametrize("heads,rank", [(4, 128), (17, 64), (2, 192), (3, 256), (2, 400), (2, 512), (5, 96), (1, 260)])
def test_latent_attention_exact_and_wide_latents(env, heads, rank):
    layers = [C.L(0, heads=heads, dim=32, vdim=24, kv_rank=rank, scale=0.2)]
    got, want, _, _ = K.run_mixer(env, layers, 200, [150, 1, 1, 40] + [1] * 8, seed=heads, width=48)
    env.close(got, want)


def test_window_edge_shows_with_one_loud_value(env):
    whole = K.check_window_edge(env)
    steps = K.check_window_edge(env, cuts=[11] + [1] * 29)
    if env.dtype == torch.float32:
        env.close(steps, whole.double().cpu().numpy(), 1e-3)
    K.check_window_edge(env, window=16, T=60, loud=16, cuts=[3, 2, 11, 15] + [1] * 29)
    K.check_window_edge(env, window=23, T=80, loud=0, cuts=[22, 2, 22, 1, 1, 1, 31])
    K.check_window_edge(env, window=140, T=430, loud=100, cuts=[230] + [1] * 200)    # windows longer than a decode split
    K.check_window_edge(env, window=128, T=430, loud=128, cuts=[250, 10] + [1] * 170)


@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_far_key_among_hundreds(env, kind):
    K.check_far_key(env, kind)
    K.check_far_key(env, kind, cuts=[285] + [1] * 15)
    K.check_far_key(env, kind, i=289, j=15, cuts=[16, 100, 2, 140] + [1] * 42)
    K.check_far_key(env, kind, i=270, j=128, cuts=[128, 130] + [1] * 42)     # the first key of a decode split
    K.check_far_key(env, kind, i=270, j=127, cuts=[129, 129] + [2] * 21)


# ------------------------------------------------------------------ HIP ops against their fp32 references
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("kind", ["silu", "gelu_tanh"])
def test_gated_act(dtype, kind):
    ops = K.Env("hip", "cuda").ops
    for rows, n in ((5, 300), (3, 301), (130, 1028), (70000, 4)):
        x = (torch.randn(rows, 2 * n) * 3).to(dtype).to(DEV)
        torch.testing.assert_close(ops.gated_act(x, kind).float(), ref.gated_act(x, kind).float(), **_tol(dtype))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("kind", ["sigmoid", "silu"])
def test_gates_per_head_and_per_feature(dtype, kind):
    """On and off the 4-column grid; the gate a column range of a wider row at aligned and odd offsets."""
    ops = K.Env("hip", "cuda").ops
    for rows, heads, vd, off, pad in ((5, 3, 20, 4, 8), (9, 5, 7, 3, 1), (130, 16, 128, 8, 0), (70001, 2, 4, 1, 3)):
        x = torch.randn(rows, heads * vd).to(dtype).to(DEV)
        for group in (vd, 1):
            w = heads * vd // group
            gate = (torch.randn(rows, off + w + pad) * 2).to(dtype).to(DEV)[:, off:off + w]
            torch.testing.assert_close(ops.gate_mul(x, gate, kind, group).float(), ref.gate_mul(x, gate, kind, group).float(), **_tol(dtype))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("H,G,d,pad", [(4, 2, 16, 4), (3, 3, 10, 3), (2, 1, 72, 0), (6, 2, 20, 8), (5, 1, 7, 1), (8, 2, 128, 16)])
def test_keys_as_values_norms_and_temperature(dtype, H, G, d, pad):
    """The write without rotation: element and 4-feature forms, small and large steps; slots of large
    steps start inside and at the edge of 4-key groups, jump, repeat pages and are out of order."""
    ops = K.Env("hip", "cuda").ops
    g = torch.Generator().manual_seed(H * d)
    BS, NB = 16, 140
    qn, kn = 1 + 0.3 * torch.randn(H * d, generator=g), 1 + 0.3 * torch.randn(G * d, generator=g)
    none = torch.empty(0)
    for T, first in ((37, 5), (1100, 3), (1100, 16), (1027, None)):
        x = torch.randn(T, (H + G) * d + pad, generator=g).to(dtype)
        pos = torch.arange(T, dtype=torch.int32) if first is not None else torch.randint(0, 5000, (T,), generator=g, dtype=torch.int32)
        slots = torch.arange(first, first + T) + BS if first is not None else torch.randperm((NB - 1) * BS, generator=g)[:T] + BS
        if first is not None and T > 1000:
            slots[501:] += 33    # a jump inside a 4-token group
        slots = slots.to(torch.int32)
        kc, vc = torch.zeros(NB, G, BS, d, dtype=dtype), torch.zeros(NB, G, d, BS, dtype=dtype)
        kd, vd = kc.to(DEV), vc.to(DEV)
        args = (H, G, d, d)
        for temp in ((0.7, 9), None):
            want = ref.rope_pairs_kv_write(x, pos, slots, *args, qn, kn, 1e-5, none, None, kc, vc, True, temp)
            got = ops.rope_pairs_kv_write(x.to(DEV), pos.to(DEV), slots.to(DEV), *args, qn.to(DEV), kn.to(DEV), 1e-5, none.to(DEV), None,
                                          kd, vd, v_is_k=True, q_temp=temp)
            torch.testing.assert_close(got.cpu().float(), want.float(), **_tol(dtype))
        kl, vl = ops.kv_to_logical(kd, vd)
        torch.testing.assert_close(kl.cpu().float(), kc.float(), **_tol(dtype))
        assert torch.equal(vl.cpu(), vc)   # values are copied


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("H,G,dim,vdim,window,cap,slopes", [
    (4, 2, 32, 32, 100, 5.0, True), (4, 2, 48, 48, 0, 30.0, True), (8, 2, 64, 64, 150, 0.0, True), (6, 6, 96, 96, 33, 2.0, False),
    (16, 4, 128, 128, 512, 30.0, True), (2, 1, 192, 192, 128, 8.0, True), (2, 2, 256, 256, 0, 8.0, True), (3, 1, 20, 18, 40, 4.0, True),
    (2, 2, 7, 5, 0, 3.0, True), (4, 1, 80, 80, 16, 9.0, True), (2, 1, 300, 272, 70, 6.0, True), (40, 2, 32, 48, 90, 6.0, True),
    (4, 1, 16, 300, 0, 0.0, False), (3, 1, 512, 512, 200, 0.0, False)])
def test_capped_and_biased_scores(dtype, H, G, dim, vdim, window, cap, slopes):
    """A packed step (portions beside single rows) and a decode step against the reference, every
    replay of the captured decode step against the eager one."""
    ops = K.Env("hip", "cuda").ops
    lens, q_lens = [700, 65, 1, 330, 129, 18], [130, 65, 1, 1, 1, 2]
    k, v, meta, T = _paged(lens, q_lens, 16, G, dim, vdim, dtype, seed=H + dim)
    g = torch.Generator().manual_seed(dim)
    q = torch.randn(T, H, dim, generator=g).to(dtype).to(DEV)
    sl = ref.alibi_slopes(H, DEV) if slopes else None
    args = (2.0 * dim ** -0.5, 1, 0.0, -1.0, 1.0, vdim, window, None, 0, cap, sl)
    kp, vp = ops.kv_from_logical(k, v)
    want = ref.multimap_attention(q, k, v, meta.block_tables, meta.q_start, meta.seq_lens, *args)
    got = ops.multimap_attention(q, kp, vp, meta, *args)
    torch.testing.assert_close(got.float(), want.float(), **(_tol(dtype) if dtype == torch.bfloat16 else dict(atol=1e-4, rtol=1e-4)))
    B = len(lens)
    last = (meta.q_start[1:] - 1).long()
    qd = q.index_select(0, last).contiguous()
    meta.decode = True
    got_d = ops.multimap_attention(qd, kp, vp, meta, *args)
    torch.testing.assert_close(got_d.float(), want.index_select(0, last).float(),
                               **(_tol(dtype) if dtype == torch.bfloat16 else dict(atol=1e-4, rtol=1e-4)))
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        ops.multimap_attention(qd, kp, vp, meta, *args)
    torch.cuda.current_stream().wait_stream(side)
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        out = ops.multimap_attention(qd, kp, vp, meta, *args)
    for i in range(3):
        qd.copy_(torch.roll(qd, 1, 0))
        eager = ops.multimap_attention(qd, kp, vp, meta, *args)
        graph.replay()
        torch.cuda.synchronize()
        assert torch.equal(out, eager) and out.shape == (B, H * vdim)


# ------------------------------------------------------------------ the engine
@pytest.fixture(scope="module", params=[(n, d) for n in C.CASES for d in DTYPES], ids=lambda p: f"{p[0]}-{p[1]}")
def case(request, tmp_path_factory):
    name, dtype = request.param
    path = str(tmp_path_factory.mktemp(name))
    cfg = C.CASES[name]
    sd = O.to_f64(C.checkpoint(cfg, path, seed=len(name)))
    e = K.Env("hip", "cuda", getattr(torch, dtype))
    e.measure_noise(path, cfg, sd)
    eng = C.engine(path, backend="hip", dtype=e.dtype, pool_tokens=320)
    assert eng.ops.name == "hip"
    yield e, cfg, sd, eng
    eng.shutdown()


def test_whole_prompt_every_position(case):
    K.whole_prompt(*case, n=150)


def test_residual_stream_after_every_layer(case):
    K.stream_after_every_layer(*case)


def test_prefill_then_token_by_token(case):
    K.prefill_then_token_by_token(*case, n=140, first=75)


def test_first_tokens_one_by_one(case):
    K.first_tokens_one_by_one(*case)


@pytest.mark.parametrize("sizes", [[2, 2, 3, 17, 16, 1, 31, 2, 5], [15, 1, 1, 16, 33, 11], [2, 3, 64, 1, 17, 2, 1, 70]])
def test_portions_of_changing_size(case, sizes):
    K.portions(*case, sizes)


def test_mixed_batches_and_reuse(case):
    K.mixed_batches_and_reuse(*case)


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation(tmp_path, graphs):
    cfg = C.CASES["mixed"]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=2))
    eng = C.engine(path, backend="hip", dtype=torch.float32, rows=4, use_hip_graphs=graphs, precapture_graphs=False)
    try:
        K.greedy_generation(K.Env("hip", "cuda"), cfg, sd, eng, tie=0.05)
    finally:
        eng.shutdown()


@pytest.mark.parametrize("graphs", [False, True])
def test_prompts_share_cached_prefixes(tmp_path, graphs):
    cfg = C.CASES["mixed"]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=2))
    eng = C.engine(path, backend="hip", dtype=torch.float32, pool_tokens=640, prefix_caching=True, prefill_chunk_tokens=24,
                   use_hip_graphs=graphs, precapture_graphs=False)
    try:
        K.shared_prefixes(K.Env("hip", "cuda"), cfg, sd, eng, tie=0.05)
    finally:
        eng.shutdown()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(10))
def test_drawn_configurations(tmp_path, seed, dtype):
    K.drawn_configuration(K.Env("hip", "cuda", getattr(torch, dtype)), tmp_path, seed)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_context_windows_across_decode_splits(tmp_path, dtype):
    """Windows longer than a decode split and a context several windows long; the latent layers read
    every key of it."""
    cfg = C.config([C.A(heads=4, kv_heads=2, dim=32, window=200, softcap=20.0, temp=(0.3, 100), scale=0.2), C.L(heads=4, kv_rank=64),
                    C.A(ff=0, heads=2, kv_heads=2, dim=16, window=131, softcap=6.0), C.L(heads=2, dim=16, vdim=32, kv_rank=64, kv_from=1)],
                   width=64, vocab=80, max_positions=1024)
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=11))
    e = K.Env("hip", "cuda", getattr(torch, dtype))
    e.measure_noise(path, cfg, sd, n=600)
    eng = C.engine(path, backend="hip", dtype=e.dtype, pool_tokens=1024, max_len=1024)
    try:
        toks = C.tokens(700, cfg["vocab"], 3)
        want = O.forward(sd, cfg, toks)
        idx = list(range(0, 520, 7)) + [519]
        e.close(eng.stream_step([("x", toks[:520], idx)]), want[idx])
        got = [eng.stream_step([("x", toks[p:p + 1], [0])]) for p in range(520, 600)]
        e.close(torch.cat(got), want[520:600])
        e.close(eng.stream_step([("x", toks[600:], list(range(100)))], end=["x"]), want[600:])
    finally:
        eng.shutdown()
