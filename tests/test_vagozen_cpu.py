"""Vagozen on the torch backend (CPU, fp32) against the float64 oracle (tests/vagozen_oracle.py):
mechanisms one by one, then the engine's packed steps, paging, state rows and generation."""
import math

import numpy as np
import pytest
import torch

import vagozen_cases as C
import vagozen_checks as K
import vagozen_oracle as O
from byzantine_consensus_llm_agents_amd.models.config import VagozenConfig, from_hf_config
from byzantine_consensus_llm_agents_amd.ops.reference import ramp_inv_freq

ENV = K.Env("torch", "cpu")


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("W", [44, 33, 256])
def test_stream_norms_and_entries(W):
    K.check_stream(ENV, W)


FEED_FORWARD = {"dense": (C.dense(24, 1.5), 40), "dense-odd": (C.dense(41, 0.7), 33), "experts": (C.moe(16, 5, 2, 1.5), 40),
                "experts-odd": (C.moe(23, 9, 4, 0.8), 33), "one-expert": (C.moe(24, 1, 1, 1.0), 32), "all-experts": (C.moe(32, 3, 3, 1.0), 32)}


@pytest.mark.parametrize("name", list(FEED_FORWARD))
def test_feed_forward(name):
    K.check_feed_forward(ENV, *FEED_FORWARD[name])


MIXERS = {
    "gqa": C.A(),
    "mha-window-7": C.A(heads=2, kv_heads=2, dim=24, vdim=30, window=7, keep=2),
    "no-window": C.A(heads=3, kv_heads=1, dim=8, vdim=8, window=0, dims=8),
    "window-1": C.A(heads=2, kv_heads=1, window=1, keep=0),
    "window-1-keep-1": C.A(heads=2, kv_heads=1, window=1, keep=1),
    "window-of-a-page": C.A(window=16, keep=16),
    "keep-beyond-the-window": C.A(window=5, keep=23),
    "keep-beyond-the-prompt": C.A(window=5, keep=90),
    "plain-rotary": C.A(scaling=None, dims=16, dim=16),
    "no-rotary": C.A(dims=0, scaling=None),
    "one-head": C.A(heads=1, kv_heads=1, vdim=31),
    "off-grid": C.A(heads=5, kv_heads=1, dim=38, vdim=37, window=17, keep=5, dims=6),
    "wide-head": C.A(heads=2, kv_heads=2, dim=70, vdim=68, window=16, keep=3, dims=70, scale=0.1),
    "many-heads": C.A(heads=17, kv_heads=1, window=30),
    "retention": C.R(),
    "retention-one-head": C.R(heads=1, dim=8, vdim=40, decay=[0.97], dims=4),
    "retention-decay-0-1": C.R(heads=2, decay=[0.0, 1.0]),
    "retention-odd": C.R(heads=4, dim=22, vdim=9, dims=6),
    "retention-wide": C.R(heads=2, dim=72, vdim=70, decay=[0.5, 0.999], dims=72),
    "retention-no-rotary": C.R(dims=0),
    "latent": C.L(),
    "latent-one-head": C.L(heads=1, dim=7, rot_dim=2, vdim=30, kv_rank=16),
    "latent-square": C.L(heads=4, dim=16, rot_dim=16, vdim=16, q_rank=16, kv_rank=16),
    "latent-odd": C.L(heads=5, dim=33, rot_dim=10, vdim=9, q_rank=7, kv_rank=75),
}


@pytest.mark.parametrize("name", list(MIXERS))
def test_mixer_whole_and_in_portions(name):
    for cuts in (None, [2, 14, 1, 1, 17, 2, 8]):
        got, want, _, _ = K.run_mixer(ENV, MIXERS[name], 45, cuts, seed=3)
        ENV.close(got, want)


def test_oracle_pieces_by_hand():
    """Closed forms of the position-dependent pieces."""
    see = lambda m, i: np.nonzero(O.sees(m, i, 12))[0].tolist()  # noqa: E731
    m = {"size": 3, "keep_first": 2}
    assert see(m, 0) == [0] and see(m, 1) == [0, 1] and see(m, 4) == [0, 1, 2, 3, 4] and see(m, 5) == [0, 1, 3, 4, 5]
    assert see(m, 11) == [0, 1, 9, 10, 11] and see(None, 3) == [0, 1, 2, 3] and see({"size": 1, "keep_first": 0}, 7) == [7]
    f, amp = O.frequencies({"dims": 8, "base": 100.0})
    assert f == pytest.approx([1.0, 10 ** -0.5, 0.1, 10 ** -1.5]) and amp == 1.0
    x = np.zeros((3, 4))
    x[:, 0] = 1.0
    t = O.turn(x, {"dims": 4, "base": 1.0}, "pairs")
    assert t[2] == pytest.approx([math.cos(2), math.sin(2), 0, 0])
    t = O.turn(x, {"dims": 4, "base": 1.0}, "halves")
    assert t[2] == pytest.approx([math.cos(2), 0, math.sin(2), 0])
    assert O.clamped_glu(np.array([9.0, -9.0]), np.array([9.0, -9.0]), 2.0) == pytest.approx(
        [2.0 * O.sigmoid(3.404) * 3.0, -9.0 * O.sigmoid(-15.318) * -1.0])
    m = {"decay": [0.5]}
    S = list(O.retention_states(m, np.array([[[2.0]], [[3.0]]]), np.array([[[1.0]], [[4.0]]])))
    assert S[0][0, 0, 0] == 2.0 and S[1][0, 0, 0] == 13.0
    runs = O.schedule({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}})
    assert runs == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]


@pytest.mark.parametrize("dims,base,scaling", [(48, 20000.0, (6.0, 384, 24.0, 2.0)), (12, 3000.0, (3.0, 64, 8.0, 1.0)), (6, 100.0, (8.0, 16, 32.0, 0.5)),
                                               (2, 10.0, (2.0, 4096, 1.0, 64.0)), (16, 1e6, None)])
def test_ramped_frequencies(dims, base, scaling):
    got, amp = ramp_inv_freq(dims, base, scaling)
    want, wamp = O.frequencies(C.rotary(dims, base, scaling))
    np.testing.assert_allclose(got.double().numpy(), want, rtol=1e-6)
    assert amp == pytest.approx(wamp)


def _with(layer, **kw):
    out = dict(layer, mixer=dict(layer["mixer"], **kw))
    return out


def _other_turn(swap=False, plain=False):
    real = O.turn

    def turn(x, rot, layout):
        if plain and rot:
            rot = {k: v for k, v in rot.items() if k != "scaling"}
        return real(x, rot, ("halves" if layout == "pairs" else "pairs") if swap else layout)
    return turn


ATT = C.A(heads=4, kv_heads=2, dim=12, vdim=8, window=12, keep=3, dims=8, scale=0.6)
RET = C.R(heads=2, dim=12, vdim=8, decay=[0.8, 0.97], dims=8)
LAT = C.L(heads=2, dim=12, rot_dim=8, scale=0.6)
MISTAKES = {
    "window one longer": (ATT, _with(ATT, mask={"size": 13, "keep_first": 3}), None),
    "window one shorter": (ATT, _with(ATT, mask={"size": 11, "keep_first": 3}), None),
    "one more kept": (ATT, _with(ATT, mask={"size": 12, "keep_first": 4}), None),
    "one fewer kept": (ATT, _with(ATT, mask={"size": 12, "keep_first": 2}), None),
    "none kept": (ATT, _with(ATT, mask={"size": 12, "keep_first": 0}), None),
    "attention in halves": (ATT, ATT, ("turn", _other_turn(swap=True))),
    "unscaled frequencies": (ATT, ATT, ("turn", _other_turn(plain=True))),
    "retention in pairs": (RET, RET, ("turn", _other_turn(swap=True))),
    "latent in halves": (LAT, LAT, ("turn", _other_turn(swap=True))),
    "decays swapped": (RET, _with(RET, decay=[0.97, 0.8]), None),
    "heads not normed": (RET, RET, ("unit_rms", lambda x, eps: x)),
    "wrong scale": (LAT, _with(LAT, scale=0.55), None),
}


@pytest.mark.parametrize("name", list(MISTAKES))
def test_a_misread_mixer_shows(name, monkeypatch):
    """A wrong reading of each mechanism, planted in the oracle, moves the output far beyond the tolerance."""
    layer, other, patch = MISTAKES[name]
    got, want, sd, h = K.run_mixer(ENV, layer, 40, None, seed=3)
    ENV.close(got, want)
    if patch:
        monkeypatch.setattr(O, *patch)
    assert np.abs(O.mixer(sd, "l0.mix.", other, h, 1e-5) - want).max() > 20 * 5e-4


def test_a_bias_left_out_shows():
    got, want, sd, h = K.run_mixer(ENV, ATT, 30, None, seed=3)
    for n in "qkv":
        other = dict(sd)
        other[f"l0.mix.{n}.b"] = sd[f"l0.mix.{n}.b"] * 0
        assert np.abs(O.mixer(other, "l0.mix.", ATT, h, 1e-5) - want).max() > 20 * 5e-4


LOOP_MISTAKES = {
    "embedding not added again": lambda sd, t, x, x0: x + sd["loop.step"][t],
    "embedding added in the first pass too": lambda sd, t, x, x0: x + x0 + sd["loop.step"][t],
    "one vector for all passes": lambda sd, t, x, x0: (x if t == 0 else x + x0) + sd["loop.step"][0],
    "no vectors": lambda sd, t, x, x0: x if t == 0 else x + x0,
    "no vector in the first pass": lambda sd, t, x, x0: x if t == 0 else x + x0 + sd["loop.step"][t],
}


@pytest.mark.parametrize("name", list(LOOP_MISTAKES))
def test_a_misread_loop_shows(name, monkeypatch):
    cfg = C.CASES["middle"]
    from byzantine_consensus_llm_agents_amd.models.vagozen import VagozenModel
    sd = O.to_f64(VagozenModel(VagozenConfig.from_dict(cfg, "t"), None, "cpu").random_state_dict(1, std=0.12))
    toks = C.tokens(12, cfg["vocab"], 1)
    want = O.forward(sd, cfg, toks)
    monkeypatch.setattr(O, "enter_pass", LOOP_MISTAKES[name])
    assert np.abs(O.forward(sd, cfg, toks) - want).max() > 20 * 5e-4


def test_window_edge_and_kept_keys_show_with_one_loud_value():
    whole = K.check_window_edge(ENV)
    steps = K.check_window_edge(ENV, cuts=[11] + [1] * 29)   # the edge is decoded alone
    ENV.close(steps, whole.double().numpy(), 2e-2)
    K.check_window_edge(ENV, window=16, T=60, loud=16, keep=2, cuts=[3, 2, 11, 15] + [1] * 29)   # edges on page borders
    K.check_window_edge(ENV, window=23, T=80, loud=5, keep=5, cuts=[22, 2, 22, 1, 1, 1, 31])     # the first token that is not kept
    K.check_window_edge(ENV, window=23, T=80, loud=4, keep=5, cuts=[22, 2, 22, 1, 1, 1, 31])     # the last that is
    K.check_window_edge(ENV, window=6, T=70, loud=16, keep=17, cuts=[2, 30] + [1] * 38)          # kept, on the next page
    K.check_window_edge(ENV, window=6, T=70, loud=0, keep=1, cuts=[2] * 35)


@pytest.mark.parametrize("kind", list(K.FAR))
def test_far_key_among_hundreds(kind):
    K.check_far_key(ENV, kind)
    K.check_far_key(ENV, kind, cuts=[285] + [1] * 15)
    K.check_far_key(ENV, kind, i=289, j=15, cuts=[16, 100, 2, 140] + [1] * 42)
    K.check_far_key(ENV, kind, T=140, i=130, j=0, cuts=[2] * 70)


def test_state_rows_are_carried_and_given_back_clean():
    """A sequence in portions, between portions of another one; a new sequence in a used row."""
    layer = C.R(heads=2, decay=[0.999, 0.9])
    model, sd = K._model(ENV, [layer], 40, 1)
    model.load_hf_state_dict(sd)
    sd64 = O.to_f64(sd)
    g = torch.Generator().manual_seed(9)
    ha, hb, hc = (K.rand_bf16(g, n, 40) for n in (30, 20, 8))
    wa, wb, wc = (O.mixer(sd64, "l0.mix.", layer, x.double().numpy(), 1e-5) for x in (ha, hb, hc))
    state = model.alloc_state(3)["runs"][0]
    state.fill_(7.0)

    def run(parts):
        meta = C.segments([(at, n) for _, _, at, n in parts], [r for _, r, _, _ in parts])
        y = model._retention(model.cfg.layers[0].mixer, model.layers[0], torch.cat([x[at:at + n] for x, _, at, n in parts]), meta, state, None)
        return torch.split(y, [n for _, _, _, n in parts])
    a1, b1 = run([(ha, 2, 0, 13), (hb, 0, 0, 2)])
    b2, a2 = run([(hb, 0, 2, 17), (ha, 2, 13, 1)])
    (a3,) = run([(ha, 2, 14, 16)])
    c1, b3 = run([(hc, 2, 0, 8), (hb, 0, 19, 1)])
    ENV.close(torch.cat([a1, a2, a3]), wa)
    ENV.close(torch.cat([b1, b2, b3]), wb)
    ENV.close(c1, wc)
    assert bool((state[1] == 7.0).all())


def test_config_round_trip(tmp_path):
    for name, cfg in C.CASES.items():
        path = str(tmp_path / name)
        C.checkpoint(cfg, path)
        read = from_hf_config(path)
        assert isinstance(read, VagozenConfig) and read.family == "vagozen" and read.tie_embeddings
        assert VagozenConfig.from_dict(read.to_dict(), "x") == VagozenConfig.from_dict(cfg, "x")
        assert read.num_params() > 0
        want = O.schedule(cfg)
        assert read.layer_runs == tuple(i for i, _ in want) and read.num_layers == len(want)
        assert read.pass_starts == {r: t for r, (_, t) in enumerate(want) if t is not None}
    for bad in ([C.A(heads=3, kv_heads=2)], [C.A(dims=18)], [C.A(dims=7)], [C.R(decay=[0.5])], [dict(C.A(), type="mlstm")],
                [C.A(dict(C.dense(), kind="glu"))], [C.A(C.moe(top=6))], [C.A(C.dense(limit=0.0))], [C.L(rot_dim=5)]):
        with pytest.raises(ValueError):
            VagozenConfig.from_dict(C.config(bad))
    for loop in ((0, 3, 1), (2, 1, 1), (0, 1, 0)):
        with pytest.raises(ValueError):
            VagozenConfig.from_dict(C.config([C.A(), C.A()], loop=loop))


# ------------------------------------------------------------------ the engine
@pytest.fixture(scope="module", params=list(C.CASES))
def case(request, tmp_path_factory):
    path = str(tmp_path_factory.mktemp(request.param))
    cfg = C.CASES[request.param]
    sd = O.to_f64(C.checkpoint(cfg, path, seed=len(request.param)))
    eng = C.engine(path, pool_tokens=320)
    yield cfg, sd, eng
    eng.shutdown()


def test_whole_prompt_every_position(case):
    K.whole_prompt(ENV, *case)


def test_residual_stream_after_every_layer(case):
    K.stream_after_every_layer(ENV, *case)


def test_prefill_then_token_by_token(case):
    K.prefill_then_token_by_token(ENV, *case)


def test_first_tokens_one_by_one(case):
    K.first_tokens_one_by_one(ENV, *case)


@pytest.mark.parametrize("sizes", [[2, 2, 3, 17, 16, 1, 31, 2, 5], [15, 1, 1, 16, 33, 11]])
def test_portions_of_changing_size(case, sizes):
    K.portions(ENV, *case, sizes)


def test_mixed_batches_equal_each_alone_and_reuse_pages_and_rows(case):
    K.mixed_batches_and_reuse(ENV, *case)


def test_long_decoding(case):
    cfg, sd, eng = case
    toks = C.tokens(150, cfg["vocab"], 6)
    want = O.forward(sd, cfg, toks)
    eng.stream_step([("l", toks[:4], [])])
    for p in range(4, 150):
        got = eng.stream_step([("l", toks[p:p + 1], [0])], end=["l"] if p == 149 else [])
        if p % 9 == 0 or p > 140:
            ENV.close(got, want[p:p + 1])


def test_greedy_generation_through_the_scheduler(case):
    K.greedy_generation(ENV, *case)


@pytest.mark.parametrize("name", ["stateless", "middle"])
def test_prompts_share_cached_prefixes_without_recurrent_layers(tmp_path, name):
    cfg = C.CASES[name]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=2))
    eng = C.engine(path, pool_tokens=640, prefix_caching=True, prefill_chunk_tokens=24)
    try:
        assert eng.model.has_seq_state == (name == "middle")
        K.shared_prefixes(ENV, cfg, sd, eng)
    finally:
        eng.shutdown()


def test_generate_command_line(tmp_path, capsys):
    from byzantine_consensus_llm_agents_amd.engine.generate import main
    cfg = C.CASES["middle"]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=6))
    prompts = [C.tokens(7, cfg["vocab"], 1), C.tokens(20, cfg["vocab"], 2)]
    argv = ["--weights", path, "--backend", "torch", "--dtype", "float32", "--max-tokens", "3", "--max-model-len", "64"]
    for p in prompts:
        argv += ["--prompt", " ".join(map(str, p))]
    assert main(argv) == 0
    lines = [l for l in capsys.readouterr().out.strip().splitlines() if l.strip()]
    assert len(lines) == 2
    for p, line in zip(prompts, lines):
        ids = [int(t) for t in line.split()]
        assert len(ids) == 3 and ids[0] == int(O.forward(sd, cfg, p)[-1].argmax())


def test_text_entry_point_with_id_prompts(tmp_path):
    from byzantine_consensus_llm_agents_amd.engine import LLM, SamplingParams
    cfg = C.CASES["start"]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=4))
    llm = LLM(path, backend="torch", weights=path, seed=1, max_model_len=128, kv_cache_gb=0.01, max_batch_seqs=4, dtype=torch.float32)
    try:
        prompt = C.tokens(12, cfg["vocab"], 8)
        out = llm.generate(" ".join(map(str, prompt)), SamplingParams(temperature=0.0, max_tokens=5))[0].outputs[0].text
        ids = [int(t) for t in out.split()]
        assert len(ids) == 5 and ids[0] == int(O.forward(sd, cfg, prompt)[-1].argmax())
    finally:
        llm.shutdown()


@pytest.mark.parametrize("seed", range(10))
def test_drawn_configurations(tmp_path, seed):
    K.drawn_configuration(ENV, tmp_path, seed)


def test_trace_replay_command(tmp_path):
    """bin/trace_run over a small trace: the logits of the wanted places, pages and rows given back."""
    import json
    import os
    import subprocess
    import sys
    cfg = C.CASES["middle"]
    path, out = str(tmp_path / "m"), str(tmp_path / "out")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=9))
    a, b = C.tokens(30, cfg["vocab"], 1), C.tokens(25, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:], "want": []}, {"id": "b", "tokens": b[:1], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": b[1:], "want": [2, 23]}], "end": ["b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", out,
                        "--max-tokens", "64", "--backend", "torch"], input="".join(json.dumps(s) + "\n" for s in steps),
                       text=True, capture_output=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = O.forward(sd, cfg, a), O.forward(sd, cfg, b)
    for name, want in (("0", wa[[0, 19]]), ("2", wb[[3, 24]])):
        got = np.fromfile(os.path.join(out, name + ".f32"), "<f4").reshape(2, -1)
        np.testing.assert_allclose(got, want, atol=5e-4, rtol=5e-4)
    assert not os.path.exists(os.path.join(out, "1.f32"))
