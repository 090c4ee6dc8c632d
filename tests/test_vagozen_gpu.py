"""Vagozen on the HIP backend against the float64 oracle: every mechanism's kernels alone (fp32 and
bf16), the new HIP ops against their PyTorch fp32 references at larger shapes, packed steps of the
engine (prompt portions beside single tokens, page and row reuse), and greedy generation through the
scheduler with captured decode graphs."""
import pytest
import torch

import vagozen_cases as C
import vagozen_checks as K
import vagozen_oracle as O
from byzantine_consensus_llm_agents_amd.ops import reference as ref
from test_seqmix_kernels_gpu import _paged
from test_vagozen_cpu import FEED_FORWARD, MIXERS

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
DEV = "cuda"


@pytest.fixture(params=DTYPES)
def env(request):
    e = K.Env("hip", "cuda", getattr(torch, request.param))
    assert e.ops.name == "hip"
    return e


@pytest.fixture(params=DTYPES)
def dtype(request):
    return getattr(torch, request.param)


@pytest.fixture(scope="module")
def ops():
    return K.Env("hip", "cuda").ops


def _tol(dtype, f32=3e-5):
    return dict(atol=2e-2, rtol=2e-2) if dtype == torch.bfloat16 else dict(atol=f32, rtol=f32)


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("W", [44, 33, 256, 1030, 1029, 2048, 5000, 12288, 16384, 9001])
def test_stream_norms_and_entries(env, W):
    K.check_stream(env, W)   # every register form, on and off the 4-column grid


@pytest.mark.parametrize("name", list(FEED_FORWARD))
def test_feed_forward(env, name):
    K.check_feed_forward(env, *FEED_FORWARD[name])


@pytest.mark.parametrize("name", list(MIXERS))
def test_mixer_whole_and_in_portions(env, name):
    layer = MIXERS[name]
    if name == "retention-decay-0-1" and env.dtype == torch.bfloat16:
        pytest.skip("decay 0: a head's output is v or -v by the sign of one dot product, a rounding turns it")
    noise = 0.0
    if env.dtype == torch.bfloat16:   # unit-norm heads of small sums are steep: what rounding does to this case
        r = K.Env("torch", "cpu", torch.bfloat16)
        got, want, _, _ = K.run_mixer(r, layer, 45, None, seed=3)
        noise = float(K.row_error(got.double().numpy(), want).max())
    for cuts in (None, [2, 14, 1, 1, 17, 2, 8]):
        got, want, _, _ = K.run_mixer(env, layer, 45, cuts, seed=3)
        env.close(got, want, noise=noise)


@pytest.mark.parametrize("heads,kv,dim,vdim,window,keep", [
    (4, 2, 32, 32, 70, 5), (8, 4, 128, 128, 80, 130), (3, 1, 48, 48, 40, 17), (17, 1, 16, 16, 40, 1), (2, 2, 64, 64, 150, 16),
    (4, 4, 96, 96, 130, 33), (2, 1, 192, 192, 64, 4), (2, 2, 256, 256, 20, 300), (1, 1, 144, 72, 33, 31), (2, 1, 300, 260, 20, 6), (2, 1, 64, 128, 128, 128)])
def test_attention_exact_and_wide_heads(env, heads, kv, dim, vdim, window, keep):
    """Heads on the 16-wide MFMA grid (the straight-line instances) and off it, GQA groups above the 16
    MFMA columns, kept keys in one and several decode splits, windows longer than a split."""
    layer = C.A(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, window=window, keep=keep, dims=dim - 4, scale=0.1)
    for cuts in (None, [150, 1, 1, 40] + [1] * 8, [2, 60, 130] + [1] * 8):
        got, want, _, _ = K.run_mixer(env, layer, 200, cuts, seed=heads, width=48)
        env.close(got, want)


@pytest.mark.parametrize("heads,rank,rot", [(4, 64, 32), (17, 64, 16), (2, 128, 64), (3, 192, 64), (2, 400, 8), (2, 496, 16), (5, 90, 6)])
def test_latent_attention_exact_and_wide_latents(env, heads, rank, rot):
    layer = C.L(heads=heads, dim=32, rot_dim=rot, vdim=24, q_rank=40, kv_rank=rank, scale=0.2)
    got, want, _, _ = K.run_mixer(env, layer, 200, [150, 1, 1, 40] + [1] * 8, seed=heads, width=48)
    env.close(got, want)


@pytest.mark.parametrize("heads,dim,vdim", [(3, 32, 32), (2, 64, 100), (4, 128, 128), (2, 200, 40), (1, 256, 256), (5, 20, 7)])
def test_retention_long_and_wide(env, heads, dim, vdim):
    """Slow and fast decays over several hundred tokens, whole and in portions of many sizes."""
    layer = C.R(heads=heads, dim=dim, vdim=vdim, decay=[(0.9995, 0.5, 0.99)[h % 3] for h in range(heads)], dims=dim - dim % 4)
    noise = 0.0
    if env.dtype == torch.bfloat16:
        r = K.Env("torch", "cpu", torch.bfloat16)
        got, want, _, _ = K.run_mixer(r, layer, 330, None, seed=heads)
        noise = float(K.row_error(got.double().numpy(), want).max())
    for cuts in (None, [64, 64, 2, 126, 1, 1, 72], [5, 200, 3, 122], [329, 1]):
        got, want, _, _ = K.run_mixer(env, layer, 330, cuts, seed=heads)
        env.close(got, want, noise=noise)


def test_window_edge_and_kept_keys_show_with_one_loud_value(env):
    whole = K.check_window_edge(env)
    steps = K.check_window_edge(env, cuts=[11] + [1] * 29)
    if env.dtype == torch.float32:
        env.close(steps, whole.double().cpu().numpy(), 2e-2)
    K.check_window_edge(env, window=16, T=60, loud=16, keep=2, cuts=[3, 2, 11, 15] + [1] * 29)
    K.check_window_edge(env, window=23, T=80, loud=5, keep=5, cuts=[22, 2, 22, 1, 1, 1, 31])
    K.check_window_edge(env, window=23, T=80, loud=4, keep=5, cuts=[22, 2, 22, 1, 1, 1, 31])
    K.check_window_edge(env, window=6, T=70, loud=16, keep=17, cuts=[2, 30] + [1] * 38)
    K.check_window_edge(env, window=140, T=430, loud=100, keep=9, cuts=[230] + [1] * 200)    # windows longer than a decode split
    K.check_window_edge(env, window=128, T=430, loud=128, keep=128, cuts=[250, 10] + [1] * 170)
    K.check_window_edge(env, window=30, T=430, loud=127, keep=128, cuts=[250, 10] + [1] * 170)
    K.check_window_edge(env, window=30, T=430, loud=140, keep=141, cuts=[300] + [1] * 130)


@pytest.mark.parametrize("kind", list(K.FAR))
def test_far_key_among_hundreds(env, kind):
    K.check_far_key(env, kind)
    K.check_far_key(env, kind, cuts=[285] + [1] * 15)
    K.check_far_key(env, kind, i=289, j=15, cuts=[16, 100, 2, 140] + [1] * 42)
    if kind != "kept":
        K.check_far_key(env, kind, i=270, j=128, cuts=[128, 130] + [1] * 42)     # the first key of a decode split
        K.check_far_key(env, kind, i=270, j=127, cuts=[129, 129] + [2] * 21)


# ------------------------------------------------------------------ HIP ops against their fp32 references
def test_clamped_gate(ops, dtype):
    for rows, n in ((5, 300), (3, 301), (130, 1028), (70000, 4)):
        x = (torch.randn(rows, 2 * n) * 3).to(dtype).to(DEV)
        torch.testing.assert_close(ops.gated_act(x, "clamped_glu", 1.5).float(), ref.gated_act(x, "clamped_glu", 1.5).float(), **_tol(dtype))


@pytest.mark.parametrize("T,W,ff,E,top", [(5, 64, 32, 4, 2), (300, 128, 96, 8, 3), (2100, 128, 64, 4, 2), (70, 100, 48, 5, 5), (33, 64, 23, 3, 1), (9, 30, 16, 6, 2)])
def test_clamped_experts(ops, dtype, T, W, ff, E, top):
    """The narrow and wide LDS-staged products, the direct one, and widths off the paired-row grid."""
    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, W, generator=g).to(dtype).to(DEV)
    up = (torch.randn(E, 2 * ff, W, generator=g) * 2 * W ** -0.5).to(dtype)
    down = (torch.randn(E, W, ff, generator=g) * ff ** -0.5).to(dtype).to(DEV)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).to(torch.int32).to(DEV)
    wts = torch.rand(T, top, generator=g).to(DEV)
    paired = torch.stack([ops.moe_pair_rows(u[:ff], u[ff:]) for u in up]).contiguous().to(DEV)
    got = ops.moe_experts(h, paired, down, idx, wts, "clamped_glu", 1.2)
    want = ref.moe_experts(h, up.to(DEV), down, idx, wts, "clamped_glu", 1.2)
    torch.testing.assert_close(got, want, **_tol(dtype, 1e-4))


@pytest.mark.parametrize("H,G,d,vd,half,pad", [(4, 2, 16, 12, 8, 4), (3, 3, 10, 7, 3, 3), (2, 1, 72, 72, 30, 0), (6, 2, 20, 8, 9, 8), (5, 1, 8, 9, 1, 1), (8, 2, 128, 128, 64, 16)])
def test_pair_rotary_with_amplitude(ops, dtype, H, G, d, vd, half, pad):
    """The write with turned heads and plain values: element and 4-feature forms, small and large steps;
    slots of large steps start inside and at the edge of 4-key groups, jump, and are out of order."""
    g = torch.Generator().manual_seed(H * d)
    BS, NB = 16, 140
    inv, amp = ref.ramp_inv_freq(2 * half, 1000.0, (4.0, 64.0, 8.0, 1.0))
    for T, first in ((37, 5), (1100, 3), (1100, 16), (1027, None)):
        x = torch.randn(T, (H + G) * d + G * vd + pad, generator=g).to(dtype)
        pos = torch.arange(T, dtype=torch.int32) if first is not None else torch.randint(0, 2000, (T,), generator=g, dtype=torch.int32)
        slots = torch.arange(first, first + T) + BS if first is not None else torch.randperm((NB - 1) * BS, generator=g)[:T] + BS
        if first is not None and T > 1000:
            slots[501:] += 33    # a jump inside a 4-token group
        slots = slots.to(torch.int32)
        kc, vc = torch.zeros(NB, G, BS, d, dtype=dtype), torch.zeros(NB, G, vd, BS, dtype=dtype)
        kd, vdv = kc.to(DEV), vc.to(DEV)
        want = ref.rope_pairs_kv_write(x, pos, slots, H, G, d, vd, None, None, 1e-5, inv, None, kc, vc, amp=amp)
        got = ops.rope_pairs_kv_write(x.to(DEV), pos.to(DEV), slots.to(DEV), H, G, d, vd, None, None, 1e-5, inv.to(DEV), None, kd, vdv, amp=amp)
        torch.testing.assert_close(got.cpu().float(), want.float(), **_tol(dtype, 5e-4))   # (angles of up to 2000 radians in fp32)
        kl, vl = ops.kv_to_logical(kd, vdv)
        torch.testing.assert_close(kl.cpu().float(), kc.float(), **_tol(dtype, 5e-4))
        assert torch.equal(vl.cpu(), vc)   # values are copied


@pytest.mark.parametrize("H,d,half,off,pad", [(3, 16, 8, 0, 0), (2, 64, 32, 8, 5), (4, 20, 6, 4, 2), (1, 7, 3, 1, 1), (16, 128, 64, 0, 0), (2, 256, 128, 4, 4), (2, 12, 0, 0, 0)])
def test_retention_vectors(ops, dtype, H, d, half, off, pad):
    g = torch.Generator().manual_seed(d)
    inv, amp = ref.ramp_inv_freq(2 * half, 1e4, (2.0, 64.0, 8.0, 1.0) if half else None)
    for T in (3, 70):
        y = torch.randn(T, off + 2 * H * d + pad, generator=g).to(dtype)
        pos = torch.randint(0, 1000, (T,), generator=g, dtype=torch.int32)
        want = ref.retention_prepare(y, off, off + H * d, H, d, d ** -0.5, pos, inv, amp)
        got = ops.retention_prepare(y.to(DEV), off, off + H * d, H, d, d ** -0.5, pos.to(DEV), inv.to(DEV), amp)
        for a, b in zip(got, want):
            assert a.dtype == torch.float32
            torch.testing.assert_close(a.cpu(), b, atol=3e-4, rtol=3e-4)


@pytest.mark.parametrize("H,Gq,dim,vdim", [(3, 3, 16, 12), (4, 2, 64, 64), (2, 2, 128, 256), (6, 3, 40, 70), (2, 1, 7, 5), (3, 3, 130, 66), (2, 2, 256, 33), (1, 1, 20, 128)])
def test_fixed_decay_recurrence(ops, dtype, H, Gq, dim, vdim):
    """Segments of every kind in one packed step (single tokens, shorter and longer than the chunked form
    takes, exactly one chunk, one token past it, several), fresh and continued, over stale rows; decays of
    0 and 1 among them; the values a column range of wider rows."""
    g = torch.Generator().manual_seed(dim + vdim)
    decay = torch.tensor([(0.97, 0.0, 1.0, 0.9995, 0.5, 0.9)[h % 6] for h in range(H)])
    parts = [(5, 1), (0, 64), (9, 2), (0, 15), (3, 16), (40, 65), (0, 1), (7, 17), (100, 200), (0, 130)]
    rows = [3, 0, 7, 1, 9, 2, 8, 5, 4, 6]
    meta = C.segments(parts, rows)
    T = sum(n for _, n in parts)
    q, k = torch.randn(T, Gq, dim, generator=g), torch.randn(T, Gq, dim, generator=g) * dim ** -0.5
    y = torch.randn(T, 3 + H * vdim + 2, generator=g).to(dtype)
    S = torch.randn(12, H, dim, vdim, generator=g)
    Sd = S.to(DEV)
    want = ref.gated_state_scan(q, k, decay, y[:, 3:3 + H * vdim], None, meta, S, False)
    dev = C.segments(parts, rows, DEV)
    got = ops.gated_state_scan(q.to(DEV), k.to(DEV), decay.to(DEV), y.to(DEV)[:, 3:3 + H * vdim], None, dev, Sd, False)
    torch.testing.assert_close(got.cpu(), want, atol=2e-4, rtol=2e-4)
    torch.testing.assert_close(Sd.cpu(), S, atol=2e-4, rtol=2e-4)
    one = C.segments([(0, 300)], [5], DEV)   # one long segment alone
    S1 = torch.full((6, H, dim, vdim), 9.0)
    S1d = S1.to(DEV)
    want = ref.gated_state_scan(q[:300], k[:300], decay, y[:300, 3:3 + H * vdim], None, C.segments([(0, 300)], [5]), S1, False)
    got = ops.gated_state_scan(q[:300].to(DEV), k[:300].to(DEV), decay.to(DEV), y.to(DEV)[:300, 3:3 + H * vdim], None, one, S1d, False)
    torch.testing.assert_close(got.cpu(), want, atol=2e-4, rtol=2e-4)
    torch.testing.assert_close(S1d.cpu(), S1, atol=2e-4, rtol=2e-4)


@pytest.mark.parametrize("R,RD,half,off", [(24, 8, 4, 5), (64, 32, 16, 0), (30, 6, 2, 3), (7, 2, 1, 1)])
def test_latent_rows_turned_in_pairs(ops, dtype, R, RD, half, off):
    g = torch.Generator().manual_seed(R)
    T, BS, NB, H, D = 37, 16, 6, 3, 10
    y = torch.randn(T, off + R + RD + 3, generator=g).to(dtype)
    w, inv = torch.rand(R, generator=g) + 0.5, torch.rand(half, generator=g)
    pos, slots = torch.randint(0, 300, (T,), generator=g, dtype=torch.int32), (torch.randperm((NB - 1) * BS, generator=g)[:T] + BS).to(torch.int32)
    kc, vc = torch.zeros(NB, 1, BS, R + RD, dtype=dtype), torch.zeros(NB, 1, R, BS, dtype=dtype)
    kd, vd = kc.to(DEV), vc.to(DEV)
    ref.latent_kv_write(y, off, R, RD, w, 1e-5, pos, slots, inv, 1.1, kc, vc, True)
    ops.latent_kv_write(y.to(DEV), off, R, RD, w.to(DEV), 1e-5, pos.to(DEV), slots.to(DEV), inv.to(DEV), 1.1, kd, vd, True)
    kl, vl = ops.kv_to_logical(kd, vd)
    torch.testing.assert_close(kl.cpu().float(), kc.float(), **_tol(dtype, 2e-4))
    torch.testing.assert_close(vl.cpu().float(), vc.float(), **_tol(dtype, 2e-4))
    src = torch.randn(T, H, D + RD, generator=g).to(dtype)
    dst = torch.zeros(T, H, R + RD, dtype=dtype)
    got = ops.rope_tail(src.to(DEV), D, dst.to(DEV), R, pos.to(DEV), inv.to(DEV), 1.1, True)
    torch.testing.assert_close(got.cpu().float(), ref.rope_tail(src, D, dst, R, pos, inv, 1.1, True).float(), **_tol(dtype, 2e-4))
    big = torch.randn(9000, H, D + RD, generator=g).to(dtype)   # (one thread walks the heads)
    bpos = torch.randint(0, 300, (9000,), generator=g, dtype=torch.int32)
    bdst = torch.zeros(9000, H, R + RD, dtype=dtype)
    got = ops.rope_tail(big.to(DEV), D, bdst.to(DEV), R, bpos.to(DEV), inv.to(DEV), 1.1, True)
    torch.testing.assert_close(got.cpu().float(), ref.rope_tail(big, D, bdst, R, bpos, inv, 1.1, True).float(), **_tol(dtype, 2e-4))


@pytest.mark.parametrize("H,G,dim,vdim,window,keep,sink", [
    (4, 2, 32, 32, 100, 5, False), (4, 2, 48, 48, 7, 30, True), (8, 2, 64, 64, 150, 130, False), (6, 6, 96, 96, 33, 16, False),
    (16, 4, 128, 128, 512, 64, True), (2, 1, 192, 192, 128, 3, False), (2, 2, 256, 256, 40, 260, False), (3, 1, 20, 18, 40, 9, True),
    (2, 2, 7, 5, 1, 2, False), (4, 1, 80, 64, 16, 100, False), (2, 1, 300, 272, 70, 1, False), (40, 2, 32, 48, 90, 17, False), (4, 1, 64, 128, 129, 700, False)])
def test_window_with_kept_keys(ops, dtype, H, G, dim, vdim, window, keep, sink):
    """A packed step (portions beside single rows) and a decode step against the reference, every
    replay of the captured decode step against the eager one."""
    lens, q_lens = [700, 65, 1, 330, 129, 18], [130, 65, 1, 1, 1, 2]
    k, v, meta, T = _paged(lens, q_lens, 16, G, dim, vdim, dtype, seed=H + dim)
    g = torch.Generator().manual_seed(dim)
    q = torch.randn(T, H, dim, generator=g).to(dtype).to(DEV)
    args = (2.0 * dim ** -0.5, 1, 0.0, -1.0, 1.0, vdim, window, torch.randn(H, generator=g).to(DEV) if sink else None, 0, 0.0, None, keep)
    kp, vp = ops.kv_from_logical(k, v)
    want = ref.multimap_attention(q, k, v, meta.block_tables, meta.q_start, meta.seq_lens, *args)
    got = ops.multimap_attention(q, kp, vp, meta, *args)
    torch.testing.assert_close(got.float(), want.float(), **_tol(dtype, 1e-4))
    B = len(lens)
    last = (meta.q_start[1:] - 1).long()
    qd = q.index_select(0, last).contiguous()
    meta.decode = True
    got_d = ops.multimap_attention(qd, kp, vp, meta, *args)
    torch.testing.assert_close(got_d.float(), want.index_select(0, last).float(), **_tol(dtype, 1e-4))
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
    name, dt = request.param
    path = str(tmp_path_factory.mktemp(name))
    cfg = C.CASES[name]
    sd = O.to_f64(C.checkpoint(cfg, path, seed=len(name)))
    e = K.Env("hip", "cuda", getattr(torch, dt))
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


@pytest.mark.parametrize("name", ["middle", "start"])
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation(tmp_path, graphs, name):
    cfg = C.CASES[name]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=2))
    eng = C.engine(path, backend="hip", dtype=torch.float32, rows=4, use_hip_graphs=graphs, precapture_graphs=False)
    try:
        K.greedy_generation(K.Env("hip", "cuda"), cfg, sd, eng, tie=0.05)
    finally:
        eng.shutdown()


@pytest.mark.parametrize("graphs", [False, True])
def test_prompts_share_cached_prefixes(tmp_path, graphs):
    cfg = C.CASES["stateless"]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=2))
    eng = C.engine(path, backend="hip", dtype=torch.float32, pool_tokens=640, prefix_caching=True, prefill_chunk_tokens=24,
                   use_hip_graphs=graphs, precapture_graphs=False)
    try:
        K.shared_prefixes(K.Env("hip", "cuda"), cfg, sd, eng, tie=0.05)
    finally:
        eng.shutdown()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("seed", range(12))
def test_drawn_configurations(tmp_path, seed, dt):
    K.drawn_configuration(K.Env("hip", "cuda", getattr(torch, dt)), tmp_path, seed)


@pytest.mark.parametrize("dt", DTYPES)
def test_long_context_kept_keys_and_states(tmp_path, dt):
    """Kept keys and windows longer than a decode split, a context several windows long, slow decays; the
    latent layer reads every key of it."""
    cfg = C.config([C.A(C.dense(), heads=4, kv_heads=2, dim=32, vdim=32, window=200, keep=140, scale=0.2, dims=32, scaling=(4.0, 256, 8.0, 1.0)),
                    C.R(heads=2, dim=32, vdim=32, decay=[0.9995, 0.98], dims=32),
                    C.A(C.moe(32, 4, 2), heads=2, kv_heads=2, dim=16, vdim=16, window=60, keep=4, dims=16),
                    C.L(C.dense(24), heads=4, kv_rank=48, rot_dim=16)], width=64, vocab=80, loop=(1, 3, 2))
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=11))
    e = K.Env("hip", "cuda", getattr(torch, dt))
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
