"""Sadodra: decoder with layer norms on the sublayers' outputs only, windowed attention with capped and
distance-biased scores, and latent attention without positions.

Every layer is ``x <- x + norm1(mixer(x))``, then ``x <- x + norm2(ff(x))`` (fp32 residual stream x; the
sublayers read x itself; layer norms with weight and bias).  The embedding adds a learned vector per
position.  The config lists the layers; a layer's mixer is one of

* ``attention``: GQA without rotation over a sliding window.  q and k are RMS-normed over their whole
  projection, the values are the keys as projected (before the norm), q is multiplied by a
  temperature that grows with its position, scaled scores pass ``softcap tanh(. / softcap)`` and lose
  ``2^(-8 (h + 1) / heads) (i - j)``;
* ``latent_attention``: queries straight from the input, keys and values from one normed latent per
  token (``models/latent.py``), one sigmoid gate per head; a layer may read an earlier layer's
  latents (``kv_from``).

Feed-forward: ``down(gelu(gate x) * (up x))``.  Nothing is kept per sequence besides the paged cache,
so prompt prefixes are cached and shared as for the Llama-style decoders.

Kernel plan of one layer (HIP backend; the torch backend runs the same ops from
``ops/reference.py``):

    attention         fused GEMM [q | k] -> rope_pairs_kv_write (norms, temperature, paged K and V from
                      the k part) -> multimap_attention (one map, window, cap, slopes) -> o GEMM
    latent_attention  fused GEMM [q | dkv | g] -> latent_kv_write; head_linear (W_uk) ->
                      multimap_attention (one KV head) -> head_linear (W_uv) -> gate_mul -> o GEMM
    residual_post_norm  x += layer_norm(y), and a rounded copy of x for the next reader
    feed-forward      [gate | up] GEMM -> gated_act (gelu) -> down GEMM -> residual_post_norm

No host synchronisation anywhere: a decode step is capturable in a HIP graph.
"""

import math
from typing import Dict, List, Optional

import torch

from ..ops.reference import alibi_slopes
from .config import SadodraConfig
from .latent import latent_mixer, latent_shapes, latent_weights
from .transformer import AttnMeta, TPGroup


class SadodraModel:
    split_single_rows = True
    logits_dtype = torch.float32
    supports_cascade = False

    def __init__(self, cfg: SadodraConfig, ops, device, dtype=torch.bfloat16, tp: Optional[TPGroup] = None,
                 quant: Optional[str] = None):
        if quant is not None:
            raise ValueError("Sadodra: quantised weights are not supported")
        self.tp = tp or TPGroup()
        if self.tp.size != 1:
            raise ValueError("Sadodra: tensor parallelism is not supported")
        self.cfg, self.ops, self.device, self.dtype, self.quant = cfg, ops, torch.device(device), dtype, None
        self.layers: List[Dict[str, torch.Tensor]] = []
        self.embed = self.pos_embed = self.lm_head = self.final_norm = None
        self.n_q = max(l.mixer.heads for l in cfg.layers)
        self.n_kv = max([l.mixer.kv_heads for l in cfg.layers if l.type == "attention"] or [1])
        self.hd = max(l.mixer.dim if l.type == "attention" else l.mixer.kv_rank for l in cfg.layers)
        self.inter = max([2 * l.mlp.ff for l in cfg.layers if l.mlp] or [0])
        self.vocab_local = cfg.vocab_size
        self.prefill_tile_rows = 64
        self.empty_freq = torch.empty(0, dtype=torch.float32, device=self.device)   # (no rotary)

    # ------------------------------------------------------------- KV cache
    @staticmethod
    def _cache_shape(l):
        """(KV heads, key features, value features) of a layer's own cache, None when it borrows one."""
        m = l.mixer
        if l.type == "attention":
            return m.kv_heads, m.dim, m.dim
        return (1, m.key_width, m.kv_rank) if m.kv_from < 0 else None

    def kv_block_bytes(self, block_size: int, dtype) -> int:
        item = torch.tensor([], dtype=dtype).element_size()
        shapes = [self._cache_shape(l) for l in self.cfg.layers]
        return sum(s[0] * (s[1] + s[2]) * block_size * item for s in shapes if s)

    def alloc_kv(self, num_blocks: int, block_size: int, dtype, device=None):
        """Per layer K [NB, G, BS, key features] and V [NB, G, value features, BS]; a latent layer
        holds one KV head of latents (K and V^T), one that borrows (``kv_from``) gets the lender's
        tensors (block ids are shared by all layers: one block table per sequence)."""
        dev = device or self.device
        ks, vs = [], []
        for l in self.cfg.layers:
            shape = self._cache_shape(l)
            if shape is None:
                ks.append(ks[l.mixer.kv_from])
                vs.append(vs[l.mixer.kv_from])
                continue
            g, kd, vd = shape
            ks.append(torch.zeros(num_blocks, g, block_size, kd, dtype=dtype, device=dev))
            vs.append(torch.zeros(num_blocks, g, vd, block_size, dtype=dtype, device=dev))
        return ks, vs

    # ------------------------------------------------------------- weights
    def tensor_shapes(self) -> Dict[str, tuple]:
        """Checkpoint tensor names -> shapes."""
        c, W = self.cfg, self.cfg.hidden_size
        out = {"embed": (c.vocab_size, W), "pos": (c.max_position, W), "head": (c.vocab_size, W)}

        def norm(name):
            out.update({name: (W,), name + ".b": (W,)})
        norm("final.norm")
        for i, l in enumerate(c.layers):
            p, m, q = f"l{i}.", l.mixer, f"l{i}.mix."
            norm(p + "norm1")
            if l.type == "attention":
                out.update({q + "q": (m.q_width, W), q + "k": (m.k_width, W), q + "q.norm": (m.q_width,), q + "k.norm": (m.k_width,),
                            q + "o": (W, m.q_width)})
            else:
                out.update(latent_shapes(m, W, q))
            if l.mlp is not None:
                norm(p + "norm2")
                out.update({p + "mlp.gate": (l.mlp.ff, W), p + "mlp.up": (l.mlp.ff, W), p + "mlp.down": (W, l.mlp.ff)})
        return out

    def random_state_dict(self, seed: int = 0, std: float = 0.05) -> Dict[str, torch.Tensor]:
        """bf16-representable random weights under the checkpoint names (tests, benchmarks)."""
        gen = torch.Generator().manual_seed(seed)
        sd = {}
        for name, shape in self.tensor_shapes().items():
            r = torch.randn(shape, generator=gen)
            if name.endswith(("norm", "norm1", "norm2")):
                t = 1.0 + 0.2 * r
            elif name.endswith(".b"):
                t = r * 0.1
            elif name in ("embed", "pos"):
                t = r * (0.7 if name == "embed" else 0.4)
            elif name.endswith((".uk", ".uv")) or name == "head":
                t = r * (1.0 / math.sqrt(shape[1]))
            else:
                t = r * std
            sd[name] = t.to(torch.bfloat16)
        return sd

    def init_random(self, seed: int = 0, std: float = 0.05):
        self.load_hf_state_dict(self.random_state_dict(seed, std))

    def load_hf_state_dict(self, sd):
        """Load the checkpoint tensors (names of `tensor_shapes`).  Projections that read the same
        input are stacked into one GEMM weight."""
        c, dev, dt = self.cfg, self.device, self.dtype

        def get(name, dtype=None):
            return sd[name].to(device=dev, dtype=dtype or dt).contiguous()

        def f32(name):
            return get(name, torch.float32)

        def norm(name):
            return ("ln", f32(name), f32(name + ".b"), c.rms_eps)

        self.layers = []
        for i, l in enumerate(c.layers):
            p, m, q = f"l{i}.", l.mixer, f"l{i}.mix."
            L = {"post1": norm(p + "norm1")}
            if l.type == "attention":
                L["fused"] = torch.cat([get(q + "q"), get(q + "k")]).contiguous()
                L["q_norm"], L["k_norm"], L["o"] = f32(q + "q.norm"), f32(q + "k.norm"), get(q + "o")
                L["slopes"] = alibi_slopes(m.heads, dev)
            else:
                L.update(latent_weights(m, q, get, f32, dev))
            if l.mlp is not None:
                L["post2"] = norm(p + "norm2")
                L["up"] = torch.cat([get(p + "mlp.gate"), get(p + "mlp.up")]).contiguous()
                L["down"] = get(p + "mlp.down")
            self.layers.append(L)
        self.embed, self.pos_embed, self.lm_head = get("embed"), get("pos"), get("head")
        self.final_norm = norm("final.norm")

    def weight_bytes(self) -> int:
        def size(v):
            if torch.is_tensor(v):
                return v.numel() * v.element_size()
            return sum(size(t) for t in v) if isinstance(v, tuple) else 0
        n = sum(size(v) for L in self.layers for v in L.values())
        return n + sum(size(t) for t in (self.embed, self.pos_embed, self.lm_head, self.final_norm))

    # ------------------------------------------------------------- sublayers
    def _attention(self, m, L, h, meta, k_cache, v_cache, sel):
        ops = self.ops
        y = ops.linear(h, L["fused"])
        q = ops.rope_pairs_kv_write(y, meta.positions, meta.slots, m.heads, m.kv_heads, m.dim, m.dim, L["q_norm"], L["k_norm"],
                                    self.cfg.rms_eps, self.empty_freq, None, k_cache, v_cache, v_is_k=True,
                                    q_temp=(m.temp_coef, m.temp_every) if m.temp_every else None)
        att = ops.multimap_attention(q, k_cache, v_cache, meta, m.scale, 1, 0.0, -1.0, 1.0, m.dim, m.window, None, 0,
                                     m.softcap, L["slopes"])
        return ops.linear(att if sel is None else att.index_select(0, sel), L["o"])

    def _latent_attention(self, m, L, h, meta, k_cache, v_cache, sel):
        return latent_mixer(self.ops, m, L, h, meta, k_cache, v_cache, sel, self.cfg.rms_eps)

    def _feed_forward(self, L, h):
        ops = self.ops
        return ops.linear(ops.gated_act(ops.linear(h, L["up"]), "gelu_tanh"), L["down"])

    # ------------------------------------------------------------- forward
    def forward(self, tokens: torch.Tensor, meta: AttnMeta, k_cache, v_cache, trace: Optional[list] = None):
        """Logits (fp32) of the rows ``meta.logits_idx`` (all rows when None).  ``trace``: a list that
        receives a copy of the residual stream after every layer (debugging)."""
        ops, c, dt = self.ops, self.cfg, self.dtype
        x, h = ops.embed_position(tokens, meta.positions, self.embed, self.pos_embed, dt)
        n_layers = len(c.layers)
        for i, (spec, L) in enumerate(zip(c.layers, self.layers)):
            last = i == n_layers - 1
            sel = meta.logits_idx if last else None
            mixer = self._attention if spec.type == "attention" else self._latent_attention
            y = mixer(spec.mixer, L, h, meta, k_cache[i], v_cache[i], sel)
            if sel is not None:   # past the last mixer only the rows whose logits are asked for matter
                x = x.index_select(0, sel)
            after = self.final_norm if last else ("copy",)
            if spec.mlp is not None:
                h = ops.residual_post_norm(x, y, L["post1"], ("copy",), dt)
                h = ops.residual_post_norm(x, self._feed_forward(L, h), L["post2"], after, dt)
            else:
                h = ops.residual_post_norm(x, y, L["post1"], after, dt)
            if trace is not None:
                trace.append(x.clone())
        return ops.linear(h, self.lm_head).float()
