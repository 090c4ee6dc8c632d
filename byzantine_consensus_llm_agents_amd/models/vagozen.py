"""Vagozen: looped decoder with RMS norms before and after every sublayer, windowed attention that keeps
the first keys, retention and latent attention.

Every layer is ``x <- x + s1 * rms1b(mixer(rms1(x)))``, then ``x <- x + s2 * rms2b(ff(rms2(x)))`` (fp32
residual stream x; s1, s2 a learned scale per feature).  A span of layers runs several passes with
shared weights; ahead of every pass but the first the token's embedding is added to the stream again,
and ahead of every pass a learned vector of that pass.  Every layer run has a cache or state of its
own.  Logits are the embedding table times the normed stream, scaled.  The config lists the layers;
a layer's mixer is one of

* ``attention``: GQA with biased projections, interleaved-pair rotary with ramped frequency scaling, a
  sliding window whose queries also see the sequence's first ``keep`` keys;
* ``retention``: per head a ``dim x vdim`` state with one fixed decay, ``S_t = decay S_(t-1) + k_t v_t^T``,
  ``o_t = S_t^T q_t`` (rotate-half rotary on q and k, k over ``sqrt(dim)``), unit-RMS heads times a silu gate;
* ``latent_attention``: queries through a normed latent, keys and values from one normed latent per
  token plus one rotated key part (``models/latent.py``), no output gate.

Feed-forward: ``down(clamped_glu(gate h, up h))``, dense or ``top`` of ``experts`` such layers weighted by
the softmax over the chosen router logits.

State per sequence besides the paged cache: per retention run one fp32 matrix per head, in tables
indexed by the engine's state row; a segment that starts at position 0 starts from zero.

Kernel plan of one layer run (HIP backend; the torch backend runs the same ops from ``ops/reference.py``):

    attention         fused GEMM [q | k | v] + bias -> rope_pairs_kv_write -> multimap_attention (one map,
                      window, kept keys) -> o GEMM
    retention         fused GEMM [q | k | v | g] -> retention_prepare -> gated_state_scan (constant decay)
                      -> head_norm_gate (silu) -> o GEMM
    latent_attention  fused GEMM [dq | dkv] -> latent_kv_write; rmsnorm_cols -> uq GEMM -> head_linear
                      (W_uk) + rope_tail -> multimap_attention (one KV head) -> head_linear (W_uv) -> o GEMM
    residual_post_norm  x += s * rms(y), the entry of the next pass, and the next reader's RMS norm, one pass
                      over the row
    feed-forward      [gate | up] GEMM -> gated_act (clamped_glu) -> down GEMM, or
                      moe_route -> grouped expert GEMMs (clamped_glu in the epilogue) -> combine

No host synchronisation anywhere: a decode step is capturable in a HIP graph.
"""

import math
from typing import Dict, List, Optional

import torch

from ..ops.reference import ramp_inv_freq
from .config import VagozenConfig
from .latent import latent_mixer, latent_shapes, latent_weights
from .transformer import AttnMeta, TPGroup


class VagozenModel:
    split_single_rows = True
    logits_dtype = torch.float32
    supports_cascade = False

    def __init__(self, cfg: VagozenConfig, ops, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None,
                 quant: Optional[str] = None):
        if quant is not None:
            raise ValueError("Vagozen: quantised weights are not supported")
        self.tp = tp or TPGroup()
        if self.tp.size != 1:
            raise ValueError("Vagozen: tensor parallelism is not supported")
        self.cfg, self.ops, self.device, self.dtype, self.quant = cfg, ops, torch.device(device), dtype, None
        # recurrent state: a cached prompt prefix cannot stand in for its tokens
        self.has_seq_state = any(l.type == "retention" for l in cfg.layers)
        self.layers: List[Dict[str, torch.Tensor]] = []
        self.embed = self.lm_head = self.final_norm = self.loop_step = None
        sizes = [1]
        for l in cfg.layers:
            m = l.mixer
            sizes += [m.key_width, m.kv_rank, m.dim + m.rot_dim] if l.type == "latent_attention" else [m.dim, m.vdim]
        self.n_q, self.n_kv, self.hd = max(l.mixer.heads for l in cfg.layers), 1, max(sizes)
        self.inter = max([2 * l.mlp.ff * max(1, l.mlp.top) for l in cfg.layers if l.mlp] or [0])
        self.vocab_local = cfg.vocab_size
        self.prefill_tile_rows = 64

    # ------------------------------------------------------------- KV cache and state
    @staticmethod
    def _cache_shape(l):
        """(KV heads, key features, value features) of a layer run's cache, None for a recurrent layer."""
        m = l.mixer
        if l.type == "attention":
            return m.kv_heads, m.dim, m.vdim
        return (1, m.key_width, m.kv_rank) if l.type == "latent_attention" else None

    def _runs(self):
        return [self.cfg.layers[i] for i in self.cfg.layer_runs]

    def kv_block_bytes(self, block_size: int, dtype) -> int:
        item = torch.tensor([], dtype=dtype).element_size()
        shapes = [self._cache_shape(l) for l in self._runs()]
        return sum(s[0] * (s[1] + s[2]) * block_size * item for s in shapes if s)

    def alloc_kv(self, num_blocks: int, block_size: int, dtype, device=None):
        """Per layer run K [NB, G, BS, key features] and V [NB, G, value features, BS] (a latent layer: one
        KV head of latents), None for the retention runs (block ids are shared by all runs: one block
        table per sequence)."""
        dev = device or self.device
        ks, vs = [], []
        for l in self._runs():
            shape = self._cache_shape(l)
            if shape is None:
                ks.append(None)
                vs.append(None)
                continue
            g, kd, vd = shape
            ks.append(torch.zeros(num_blocks, g, block_size, kd, dtype=dtype, device=dev))
            vs.append(torch.zeros(num_blocks, g, vd, block_size, dtype=dtype, device=dev))
        return ks, vs

    def alloc_state(self, rows: int, device=None) -> dict:
        """State tables with ``rows`` rows, per retention run fp32 [rows, heads, dim, vdim]; None for the others."""
        dev = device or self.device
        return {"runs": [torch.zeros(rows, l.mixer.heads, l.mixer.dim, l.mixer.vdim, dtype=torch.float32, device=dev)
                         if l.type == "retention" else None for l in self._runs()]}

    @staticmethod
    def state_tensors(state: dict) -> List[torch.Tensor]:
        """Every table of `alloc_state` (row-indexed in dimension 0): what the engine moves when
        it moves a row."""
        return [t for t in state["runs"] if t is not None]

    def state_row_bytes(self) -> int:
        return sum(4 * l.mixer.heads * l.mixer.dim * l.mixer.vdim for l in self._runs() if l.type == "retention")

    # ------------------------------------------------------------- weights
    def tensor_shapes(self) -> Dict[str, tuple]:
        """Checkpoint tensor names -> shapes."""
        c, W = self.cfg, self.cfg.hidden_size
        out = {"embed": (c.vocab_size, W), "final.norm": (W,)}
        if c.pass_starts:
            out["loop.step"] = (c.loop_times, W)
        for i, l in enumerate(c.layers):
            p, m, q, f = f"l{i}.", l.mixer, f"l{i}.mix.", l.mlp
            out.update({p + n: (W,) for n in ("norm1", "norm1b", "ls1") + (("norm2", "norm2b", "ls2") if f is not None else ())})
            if l.type == "attention":
                for n, width in (("q", m.q_width), ("k", m.k_width), ("v", m.v_width)):
                    out.update({q + n: (width, W), q + n + ".b": (width,)})
                out[q + "o"] = (W, m.heads * m.vdim)
            elif l.type == "retention":
                out.update({q + "q": (m.qk_width, W), q + "k": (m.qk_width, W), q + "v": (m.v_width, W), q + "g": (m.v_width, W),
                            q + "o": (W, m.v_width)})
            else:
                out.update(latent_shapes(m, W, q))
            if f is not None:
                for e in [""] if f.kind == "dense" else [f"e{e}." for e in range(f.experts)]:
                    out.update({p + f"mlp.{e}gate": (f.ff, W), p + f"mlp.{e}up": (f.ff, W), p + f"mlp.{e}down": (W, f.ff)})
                if f.kind == "moe":
                    out.update({p + "mlp.router": (f.experts, W), p + "mlp.router.b": (f.experts,)})
        return out

    def random_state_dict(self, seed: int = 0, std: float = 0.05) -> Dict[str, torch.Tensor]:
        """bf16-representable random weights under the checkpoint names (tests, benchmarks)."""
        gen = torch.Generator().manual_seed(seed)
        sd = {}
        for name, shape in self.tensor_shapes().items():
            r = torch.randn(shape, generator=gen)
            if name.endswith(("norm", "norm1", "norm2", "norm1b", "norm2b")):
                t = 1.0 + 0.2 * r
            elif name.endswith(("ls1", "ls2")):
                t = 0.6 + 0.15 * r
            elif name.endswith("router.b"):
                t = r * 0.5
            elif name.endswith(".b") or name == "loop.step":
                t = r * 0.3
            elif name.endswith((".uq", ".uk", ".uv")):
                t = r * (1.0 / math.sqrt(shape[1]))
            elif name == "embed":
                t = r * 0.7
            elif name.endswith("router"):
                t = r * 0.3
            else:
                t = r * std
            sd[name] = t.to(torch.bfloat16)
        return sd

    def init_random(self, seed: int = 0, std: float = 0.05):
        self.load_hf_state_dict(self.random_state_dict(seed, std))

    def load_hf_state_dict(self, sd):
        """Load the checkpoint tensors (names of `tensor_shapes`).  Projections that read the same input are
        stacked into one GEMM weight, every expert's gate and up rows into one [E, 2 ff, W] tensor; a
        sublayer's output norm and its scale become one fp32 weight."""
        c, dev, dt, eps = self.cfg, self.device, self.dtype, self.cfg.rms_eps

        def get(name, dtype=None):
            return sd[name].to(device=dev, dtype=dtype or dt).contiguous()

        def f32(name):
            return get(name, torch.float32)

        pair = getattr(self.ops, "moe_pair_rows", None)
        self.layers = []
        for i, l in enumerate(c.layers):
            p, m, q, f = f"l{i}.", l.mixer, f"l{i}.mix.", l.mlp
            L = {"pre1": ("rms", f32(p + "norm1"), eps), "post1": ("rms", f32(p + "norm1b") * f32(p + "ls1"), eps)}
            if l.type == "attention":
                L["fused"] = torch.cat([get(q + n) for n in "qkv"]).contiguous()
                L["bias"] = torch.cat([get(q + n + ".b") for n in "qkv"]).contiguous()
                L["o"] = get(q + "o")
                L["inv_freq"], L["amp"] = ramp_inv_freq(m.rot_dims, m.rot_base, m.rot_scaling, dev)
            elif l.type == "retention":
                L["fused"] = torch.cat([get(q + n) for n in "qkvg"]).contiguous()
                L["o"], L["decay"] = get(q + "o"), torch.tensor(m.decay, dtype=torch.float32, device=dev)
                L["inv_freq"], L["amp"] = ramp_inv_freq(m.rot_dims, m.rot_base, m.rot_scaling, dev)
            else:
                L.update(latent_weights(m, q, get, f32, dev))
            if f is not None:
                L["pre2"], L["post2"] = ("rms", f32(p + "norm2"), eps), ("rms", f32(p + "norm2b") * f32(p + "ls2"), eps)
            if f is not None and f.kind == "dense":
                L["up"] = torch.cat([get(p + "mlp.gate"), get(p + "mlp.up")]).contiguous()
                L["down"] = get(p + "mlp.down")
            elif f is not None:
                ups = []
                for e in range(f.experts):
                    g, u = get(p + f"mlp.e{e}.gate"), get(p + f"mlp.e{e}.up")
                    ups.append(pair(g, u) if pair else torch.cat([g, u]))
                L["e_up"] = torch.stack(ups).contiguous()
                L["e_down"] = torch.stack([get(p + f"mlp.e{e}.down") for e in range(f.experts)]).contiguous()
                L["router"], L["router_b"] = f32(p + "mlp.router"), f32(p + "mlp.router.b")
            self.layers.append(L)
        self.embed = self.lm_head = get("embed")
        self.final_norm = ("rms", f32("final.norm"), eps)
        self.loop_step = f32("loop.step") if c.pass_starts else None

    def weight_bytes(self) -> int:
        def size(v):
            if torch.is_tensor(v):
                return v.numel() * v.element_size()
            return sum(size(t) for t in v) if isinstance(v, tuple) else 0
        n = sum(size(v) for L in self.layers for v in L.values())
        return n + sum(size(t) for t in (self.embed, self.final_norm, self.loop_step))

    # ------------------------------------------------------------- sublayers
    def _attention(self, m, L, h, meta, k_cache, v_cache, sel):
        ops = self.ops
        y = ops.linear(h, L["fused"], L["bias"])
        q = ops.rope_pairs_kv_write(y, meta.positions, meta.slots, m.heads, m.kv_heads, m.dim, m.vdim, None, None, self.cfg.rms_eps,
                                    L["inv_freq"], None, k_cache, v_cache, amp=L["amp"])
        att = ops.multimap_attention(q, k_cache, v_cache, meta, m.scale, 1, 0.0, -1.0, 1.0, m.vdim, m.window, keep=m.keep)
        return ops.linear(att if sel is None else att.index_select(0, sel), L["o"])

    def _retention(self, m, L, h, meta, state, sel):
        ops = self.ops
        y = ops.linear(h, L["fused"])
        n, nv = m.qk_width, m.v_width
        q32, k32 = ops.retention_prepare(y, 0, n, m.heads, m.dim, m.dim ** -0.5, meta.positions, L["inv_freq"], L["amp"])
        o32 = ops.gated_state_scan(q32, k32, L["decay"], y[:, 2 * n:2 * n + nv], None, meta, state, False)
        gate = y[:, 2 * n + nv:2 * n + 2 * nv]
        if sel is not None:
            o32, gate = o32.index_select(0, sel), gate.index_select(0, sel)
        return ops.linear(ops.head_norm_gate(o32, None, self.cfg.rms_eps, gate, self.dtype, "silu"), L["o"])

    def _latent_attention(self, m, L, h, meta, k_cache, v_cache, sel):
        return latent_mixer(self.ops, m, L, h, meta, k_cache, v_cache, sel, self.cfg.rms_eps)

    def _mixer(self, spec, L, h, meta, k_cache, v_cache, state, sel):
        if spec.type == "retention":
            return self._retention(spec.mixer, L, h, meta, state, sel)
        return (self._attention if spec.type == "attention" else self._latent_attention)(spec.mixer, L, h, meta, k_cache, v_cache, sel)

    def _feed_forward(self, f, L, h):
        ops = self.ops
        if f.kind == "dense":
            return ops.linear(ops.gated_act(ops.linear(h, L["up"]), "clamped_glu", f.limit), L["down"])
        idx, w, _ = ops.moe_route(h, L["router"], L["router_b"], f.top)
        return ops.moe_experts(h, L["e_up"], L["e_down"], idx, w, "clamped_glu", f.limit)

    # ------------------------------------------------------------- forward
    def forward(self, tokens: torch.Tensor, meta: AttnMeta, k_cache, v_cache, trace: Optional[list] = None):
        """Logits (fp32) of the rows ``meta.logits_idx`` (all rows when None).  ``meta.state`` holds the tables
        of `alloc_state`, ``meta.state_rows`` every segment's row in them.  ``trace``: a list that receives a
        copy of the residual stream after every layer run, before what enters ahead of the next pass
        (debugging)."""
        ops, c, dt = self.ops, self.cfg, self.dtype
        st = meta.state
        if self.has_seq_state and (st is None or meta.state_rows is None or meta.q_start is None or meta.token_seq is None):
            raise ValueError("Vagozen: the step carries no sequence state (state, state_rows, q_start, token_seq)")
        runs, passes = c.layer_runs, c.pass_starts
        h, x = ops.embed_scale_rmsnorm(tokens, self.embed, 1.0, self.layers[runs[0]]["pre1"][1], c.rms_eps, 0.0, dt,
                                       self.loop_step[0] if 0 in passes else None)
        for r, li in enumerate(runs):
            spec, L = c.layers[li], self.layers[li]
            last = r == len(runs) - 1
            sel = meta.logits_idx if last else None
            y = self._mixer(spec, L, h, meta, k_cache[r], v_cache[r], st["runs"][r] if st is not None else None, sel)
            if sel is not None:   # past the last mixer only the rows whose logits are asked for matter
                x = x.index_select(0, sel)
            post = L["post1"]
            if spec.mlp is not None:
                y = self._feed_forward(spec.mlp, L, ops.residual_post_norm(x, y, post, L["pre2"], dt))
                post = L["post2"]
            nxt = self.final_norm if last else self.layers[runs[r + 1]]["pre1"]
            entry = None
            if r + 1 in passes:   # the next run opens a pass: its vector, from the second pass on the embedding too
                t = passes[r + 1]
                entry = (self.loop_step[t], tokens, self.embed if t > 0 else None)
            if trace is None or entry is None:
                h = ops.residual_post_norm(x, y, post, nxt, dt, entry)
                if trace is not None:
                    trace.append(x.clone())
            else:
                ops.residual_post_norm(x, y, post, None, dt)
                trace.append(x.clone())
                h = ops.residual_post_norm(x, None, None, nxt, dt, entry)
        return ops.linear(h, self.lm_head).float() * c.logit_scale
