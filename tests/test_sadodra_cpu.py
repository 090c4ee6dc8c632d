"""Sadodra on the torch backend (CPU, fp32) against the float64 oracle (tests/sadodra_oracle.py):
mechanisms one by one, then the engine's packed steps, paging, prefix reuse and generation."""
import math

import numpy as np
import pytest
import torch

import sadodra_cases as C
import sadodra_checks as K
import sadodra_oracle as O
from byzantine_consensus_llm_agents_amd.models.config import SadodraConfig, from_hf_config

ENV = K.Env("torch", "cpu")


# ------------------------------------------------------------------ mechanisms
def test_embedding_and_layer_norms():
    for W in (44, 33, 256):
        K.check_embedding(ENV, W)
        K.check_layer_norms(ENV, W)


@pytest.mark.parametrize("W,ff", [(40, 24), (33, 41), (64, 7)])
def test_feed_forward(W, ff):
    K.check_feed_forward(ENV, W, ff)


ATTENTION = {
    "gqa": [C.A(0)],
    "mha-window-7": [C.A(0, heads=2, kv_heads=2, dim=24, window=7)],
    "one-kv-head-no-window": [C.A(0, heads=3, kv_heads=1, dim=8, window=0)],
    "window-1": [C.A(0, heads=2, kv_heads=1, window=1)],
    "window-of-a-page": [C.A(0, window=16, temp=(1.0, 1))],
    "no-cap": [C.A(0, softcap=0)],
    "tight-cap": [C.A(0, softcap=0.5, scale=2.0)],
    "no-temperature": [C.A(0, temp=None)],
    "one-head": [C.A(0, heads=1, kv_heads=1)],
    "off-grid-37": [C.A(0, heads=5, kv_heads=1, dim=37, window=37, scale=0.3)],
    "wide-head": [C.A(0, heads=2, kv_heads=2, dim=70, window=16, softcap=25.0, scale=0.1)],
    "many-heads": [C.A(0, heads=17, kv_heads=1, dim=16, window=40)],
}
LATENT = {
    "own": [C.L(0)],
    "one-head": [C.L(0, heads=1, dim=7, vdim=30, kv_rank=16)],
    "square": [C.L(0, heads=4, dim=16, vdim=16, kv_rank=16)],
    "off-grid": [C.L(0, heads=5, dim=33, vdim=9, kv_rank=75)],
    "borrowed": [C.L(0), C.L(0, heads=5, dim=9, vdim=6, kv_from=0)],
    "borrowed-past-another": [C.A(0), C.L(0, kv_rank=20), C.L(0), C.L(0, heads=2, dim=20, vdim=8, kv_rank=20, kv_from=1)],
}


@pytest.mark.parametrize("name", list(ATTENTION))
def test_attention_whole_and_in_portions(name):
    for cuts in (None, [2, 14, 1, 1, 17, 2, 8]):
        got, want, _, _ = K.run_mixer(ENV, ATTENTION[name], 45, cuts, seed=3)
        ENV.close(got, want)


@pytest.mark.parametrize("name", list(LATENT))
def test_latent_attention_whole_and_in_portions(name):
    for cuts in (None, [2, 14, 1, 1, 17, 2, 8]):
        got, want, _, _ = K.run_mixer(ENV, LATENT[name], 45, cuts, seed=3)
        ENV.close(got, want)


def test_oracle_pieces_by_hand():
    """Closed forms of the position-dependent pieces."""
    m = {"q_temp": {"coef": 0.5, "every": 4}, "heads": 4, "scale": 0.5, "softcap": 2.0}
    assert [O.temperature(m, t) for t in (0, 2)] == [1.0, 1.0]
    assert O.temperature(m, 3) == pytest.approx(1 + 0.5 * math.log(2)) == O.temperature(m, 6)
    assert O.temperature(m, 7) == pytest.approx(1 + 0.5 * math.log(3))
    assert [O.slope(h, 4) for h in range(4)] == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    s = O.scores(m, 1, np.array([1.0, 2.0]), np.array([[1.0, 0.0], [0.0, 3.0]]), 9, 5)
    assert s == pytest.approx([2 * math.tanh(0.25) - 4 / 16, 2 * math.tanh(1.5) - 3 / 16])


def _other_scores(order):
    def scores(m, h, q, keys, i, first):
        s = keys @ q * m["scale"]
        bias = O.slope(h, m["heads"]) * (i - (first + np.arange(len(keys))))
        if order == "bias inside the cap":
            return m["softcap"] * np.tanh((s - bias) / m["softcap"])
        if order == "no bias":
            return m["softcap"] * np.tanh(s / m["softcap"])
        return s - bias   # no cap
    return scores


MISTAKES = {
    "no temperature": ("temperature", lambda m, t: 1.0),
    "temperature from the position, not the next": ("temperature", lambda m, t: 1.0 + m["q_temp"]["coef"] * math.log(t // m["q_temp"]["every"] + 1)),
    "temperature without the floor": ("temperature", lambda m, t: 1.0 + m["q_temp"]["coef"] * math.log((t + 1) / m["q_temp"]["every"] + 1)),
    "slopes from head 0": ("slope", lambda h, H: 2.0 ** (-8.0 * h / H)),
    "bias inside the cap": ("scores", _other_scores("bias inside the cap")),
    "no bias": ("scores", _other_scores("no bias")),
    "no cap": ("scores", _other_scores("no cap")),
    "window one longer": ("window", 1),
    "window one shorter": ("window", -1),
    "norm per head": ("norm", None),
}


@pytest.mark.parametrize("name", list(MISTAKES))
def test_a_misread_attention_shows(name, monkeypatch):
    """A wrong reading of each mechanism, planted in the oracle, moves the output far beyond the tolerance."""
    what, new = MISTAKES[name]
    layers = [C.A(0, heads=4, kv_heads=2, dim=8, window=12, softcap=3.0, temp=(0.8, 8), scale=0.6)]
    got, want, sd, hs = K.run_mixer(ENV, layers, 40, None, seed=3)
    ENV.close(got, want)
    if what in ("temperature", "slope", "scores"):
        monkeypatch.setattr(O, what, new)
    elif what == "window":
        layers = [C.A(0, heads=4, kv_heads=2, dim=8, window=12 + new, softcap=3.0, temp=(0.8, 8), scale=0.6)]
    else:
        plain = O.rms
        monkeypatch.setattr(O, "rms", lambda x, w, eps: plain(x.reshape(len(x), -1, 8), w.reshape(-1, 8), eps).reshape(x.shape))
    assert np.abs(K.oracle_mixer(layers, sd, hs) - want).max() > 20 * 3e-4


def test_values_are_the_keys_before_their_norm():
    """Doubling the key norm's weight changes scores only: with a zero query weight it changes nothing."""
    def craft(sd, hs):
        sd["l0.mix.q.norm"] *= 0
        sd["l0.mix.k.norm"] *= 5
    got, want, sd, hs = K.run_mixer(ENV, [C.A(0, window=6)], 30, None, craft, seed=3)
    ENV.close(got, want)
    plain = dict(sd)
    plain["l0.mix.k.norm"] = sd["l0.mix.k.norm"] / 5
    np.testing.assert_allclose(K.oracle_mixer([C.A(0, window=6)], plain, hs), want, atol=1e-12)


def test_borrowed_latents_are_the_lenders():
    layers = LATENT["borrowed"]
    _, want, sd, hs = K.run_mixer(ENV, layers, 20, None, seed=3)
    own = O.latent_attention(sd, "l1.mix.", layers[1]["mixer"], hs[1], O.latent(sd, "l0.mix.", hs[1], 1e-5))
    assert np.abs(own - want).max() > 0.05   # (from the borrower's own input: another result)


def test_window_edge_shows_with_one_loud_value():
    whole = K.check_window_edge(ENV)
    steps = K.check_window_edge(ENV, cuts=[11] + [1] * 29)   # the edge is decoded alone
    ENV.close(steps, whole.double().numpy(), 1e-3)
    K.check_window_edge(ENV, window=16, T=60, loud=16, cuts=[3, 2, 11, 15] + [1] * 29)   # edges on page borders
    K.check_window_edge(ENV, window=23, T=80, loud=0, cuts=[22, 2, 22, 1, 1, 1, 31])     # the first token's last reader


@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_far_key_among_hundreds(kind):
    K.check_far_key(ENV, kind)
    K.check_far_key(ENV, kind, cuts=[285] + [1] * 15)
    K.check_far_key(ENV, kind, i=289, j=15, cuts=[16, 100, 2, 140] + [1] * 42)
    K.check_far_key(ENV, kind, T=140, i=130, j=0, cuts=[2] * 70)


def test_config_round_trip(tmp_path):
    for name, cfg in C.CASES.items():
        path = str(tmp_path / name)
        C.checkpoint(cfg, path)
        read = from_hf_config(path)
        assert isinstance(read, SadodraConfig) and read.family == "sadodra" and read.max_position == cfg["max_positions"]
        assert SadodraConfig.from_dict(read.to_dict(), "x") == SadodraConfig.from_dict(cfg, "x")
        assert read.num_params() > 0
    for bad in ([C.L(kv_from=0)], [C.A(), C.L(kv_from=0)], [C.L(), C.L(kv_from=0), C.L(kv_from=1)], [C.L(), C.L(kv_rank=9, kv_from=0)],
                [C.A(heads=3, kv_heads=2)], [dict(C.A(), type="mlstm")], [dict(C.A(), mlp={"kind": "moe"})]):
        with pytest.raises(ValueError):
            SadodraConfig.from_dict(C.config(bad))


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


def test_prompts_share_cached_prefixes(tmp_path):
    cfg = C.CASES["mixed"]
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=2))
    eng = C.engine(path, pool_tokens=640, prefix_caching=True, prefill_chunk_tokens=24)
    try:
        K.shared_prefixes(ENV, cfg, sd, eng)
    finally:
        eng.shutdown()


def test_sequences_end_at_the_last_learned_position(tmp_path):
    cfg = dict(C.CASES["latents"], max_positions=40)
    path = str(tmp_path / "m")
    sd = O.to_f64(C.checkpoint(cfg, path, seed=3))
    eng = C.engine(path, pool_tokens=256)
    try:
        assert eng.args.max_model_len == 40
        toks = C.tokens(41, cfg["vocab"], 3)
        ENV.close(eng.stream_step([("a", toks[:40], list(range(40)))], end=[]), O.forward(sd, cfg, toks[:40]))
        with pytest.raises(ValueError):
            eng.stream_step([("a", toks[40:], [0])])
        eng.stream_step([], end=["a"])
        out = eng.generate_ids([toks[:35]], 20)[0]
        assert len(out) == 5
        K.follow_greedy(cfg, sd, toks[:35], out)
    finally:
        eng.shutdown()


def test_generate_command_line(tmp_path, capsys):
    from byzantine_consensus_llm_agents_amd.engine.generate import main
    cfg = C.CASES["mixed"]
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
    cfg = C.CASES["windows"]
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


@pytest.mark.parametrize("seed", range(8))
def test_drawn_configurations(tmp_path, seed):
    K.drawn_configuration(ENV, tmp_path, seed)


def test_trace_replay_command(tmp_path):
    """bin/trace_run over a small trace: the logits of the wanted places, pages and rows given back."""
    import json
    import os
    import subprocess
    import sys
    cfg = C.CASES["mixed"]
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
        np.testing.assert_allclose(got, want, atol=3e-4, rtol=3e-4)
    assert not os.path.exists(os.path.join(out, "1.f32"))
