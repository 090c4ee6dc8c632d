"""The latent-attention mixer shared by the families that have one (Mabivik, Sadodra, Vagozen).

Keys and values are read from ONE normed latent per token, ``c = rms(W_dkv h)``, plus an optional
rotated key part shared by all heads.  The cache holds ``[c | rotated part]`` per token and the
attention runs in the latent: head h's query becomes ``[W_uk[h]^T q_h | rotated q_h]``, the
softmax-weighted sum of c is expanded by ``W_uv[h]`` afterwards, so all heads read one KV head and
nothing per head is cached.  Queries come from the input or through a normed latent of their own
(``q_rank``); the sigmoid output gate, if there is one (``gated``), has one column per value feature or
one per head (``head_gate``); the rotated part turns in halves or in neighbouring pairs
(``rot_pairs``); a layer may read an earlier layer's cache (``kv_from``) with projections of its own.
"""

import torch

from ..ops.reference import ramp_inv_freq


def latent_shapes(m, W: int, q: str) -> dict:
    """Checkpoint tensor names -> shapes of one mixer (prefix ``q``)."""
    out = {}
    if m.q_rank:
        out.update({q + "dq": (m.q_rank, W), q + "dq.norm": (m.q_rank,), q + "uq": (m.q_width, m.q_rank)})
    else:
        out[q + "q"] = (m.q_width, W)
    out.update({q + "uk": (m.heads * m.dim, m.kv_rank), q + "uv": (m.heads * m.vdim, m.kv_rank)})
    if m.gated:
        out[q + "g"] = (m.gate_width, W)
    out[q + "o"] = (W, m.heads * m.vdim)
    if m.kv_from < 0:
        out.update({q + "dkv": (m.key_width, W), q + "dkv.norm": (m.kv_rank,)})
    return out


def latent_weights(m, q: str, get, f32, device) -> dict:
    """The mixer's tensors as `latent_mixer` reads them: the projections of the input stacked into
    one GEMM weight ``[dq or q | dkv | g]`` (what there is of them), the per-head expansions as [heads, inputs, outputs]."""
    L = {"fused": torch.cat([get(q + ("dq" if m.q_rank else "q"))] + ([get(q + "dkv")] if m.kv_from < 0 else [])
                            + ([get(q + "g")] if m.gated else [])).contiguous(), "o": get(q + "o")}
    if m.q_rank:
        L["q_norm"], L["uq"] = f32(q + "dq.norm"), get(q + "uq")
    if m.kv_from < 0:
        L["kv_norm"] = f32(q + "dkv.norm")
    # per head, as right operands [inputs, outputs]: W_uk[h] (dim -> kv_rank), W_uv[h]^T (kv_rank -> vdim)
    L["uk"] = get(q + "uk").reshape(m.heads, m.dim, m.kv_rank).contiguous()
    L["uv_t"] = get(q + "uv").reshape(m.heads, m.vdim, m.kv_rank).transpose(1, 2).contiguous()
    L["inv_freq"], L["amp"] = ramp_inv_freq(m.rot_dims, m.rot_base, m.rot_scaling, device)
    return L


def latent_mixer(ops, m, L, h, meta, k_cache, v_cache, sel, eps: float):
    """The mixer's output for the input rows ``h`` (of the rows ``sel`` only when given; every row's
    latent goes to the cache)."""
    T, dt = h.shape[0], h.dtype
    y = ops.linear(h, L["fused"])
    off_g = off = m.q_rank or m.q_width
    if m.kv_from < 0:
        ops.latent_kv_write(y, off, m.kv_rank, m.rot_dim, L["kv_norm"], eps, meta.positions, meta.slots,
                            L["inv_freq"], L["amp"], k_cache, v_cache, m.rot_pairs)
        off_g += m.key_width
    if m.q_rank:
        q = ops.linear(ops.rmsnorm_cols(y, 0, m.q_rank, L["q_norm"], eps, dt), L["uq"])
    else:
        q = y[:, :m.q_width]
    q = q.view(T, m.heads, m.dim + m.rot_dim)
    qf = torch.empty(T, m.heads, m.key_width, dtype=dt, device=h.device)
    ops.head_linear(q[:, :, :m.dim], L["uk"], qf[:, :, :m.kv_rank])
    if m.rot_dim:
        ops.rope_tail(q, m.dim, qf, m.kv_rank, meta.positions, L["inv_freq"], L["amp"], m.rot_pairs)
    lat = ops.multimap_attention(qf, k_cache, v_cache, meta, m.scale, 1, 0.0, -1.0, 1.0, m.kv_rank, m.window, None)
    if sel is not None:
        lat = lat.index_select(0, sel)
    att = ops.head_linear(lat.view(-1, m.heads, m.kv_rank), L["uv_t"]).view(-1, m.heads * m.vdim)
    if m.gated:
        gate = y[:, off_g:off_g + m.gate_width]
        att = ops.gate_mul(att, gate if sel is None else gate.index_select(0, sel), "sigmoid", m.heads * m.vdim // m.gate_width)
    return ops.linear(att, L["o"])
