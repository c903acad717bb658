"""Ops of the hybrid sequence mixers: latent attention (compressed K/V cache, sliding window,
softmax sink), grouped attention over paged rows (softmax or sigmoid weights, distance penalty), the
mLSTM matrix memory, gated linear attention, the generalized delta rule, matrix memories with one decay per head and
token (gated delta rule, state-space duality, retention), differential attention, the minGRU recurrence, the
group-limited sigmoid router and the softmax router with a selection bias (optionally group-limited), and the fp32 residual stream of parallel layers, of layers with a gated residual between two norms, of layers over several
residual streams (hyper-connections), of layers whose sublayers read a causally convolved, group-normed input, and of layers whose
sublayers are normed on their way out only.

GPU tensors run the HIP kernels of ``csrc/hybrid`` (``torch.ops.llmctl_hybrid.*``, library
``_llmctl_hybrid.so``); CPU tensors run :mod:`llmctl.ops.ref_hybrid`.  All activations are
token-major ``[T, features]`` over the step's packed tokens; sequences are described by ``cu``
(row offsets, int32 [n + 1]), ``ctx`` (context length after the step, int32 [n]) and block tables.

Precision: norms, rotary angles, attention scores / softmax, the recurrence with its gates and the
residual stream are fp32 inside every kernel whatever the activation dtype (bf16 or fp32).
"""

from __future__ import annotations

import torch

from . import ref_hybrid as ref
from ._lib import native_hybrid, use_native


def layernorm_f32(x, w, b, eps: float, out_dtype):
    """LayerNorm of the fp32 residual stream ``x [T, W]`` -> ``out_dtype``."""
    if use_native(x):
        return native_hybrid().layernorm_f32(x, w, b, eps, out_dtype == torch.bfloat16)
    return ref.layernorm_f32(x, w, b, eps, out_dtype)


def residual_add_(x, a, b=None):
    """``x += a (+ b)`` on the fp32 residual stream (a, b: any float dtype)."""
    if use_native(x):
        native_hybrid().residual_add_(x, a, b)
        return x
    return ref.residual_add_(x, a, b)


def add_layernorm_f32_(x, a, b, w, bias, eps: float, out_dtype):
    """``x += a (+ b)`` in place, then LayerNorm(x) -> ``out_dtype``: the parallel layer's residual
    update and the next layer's norm in one pass over the stream."""
    if use_native(x):
        return native_hybrid().add_layernorm_f32_(x, a, b, w, bias, eps, out_dtype == torch.bfloat16)
    ref.residual_add_(x, a, b)
    return ref.layernorm_f32(x, w, bias, eps, out_dtype)


def rmsnorm_cols(x, w, eps: float, n: int, out_dtype):
    """RMS norm (weight ``w [n]``) of the first ``n`` columns of ``x [T, N]`` -> ``[T, n]``."""
    if use_native(x):
        return native_hybrid().rmsnorm_cols(x, w, eps, n, out_dtype == torch.bfloat16)
    return ref.rmsnorm_cols(x, w, eps, n, out_dtype)


def latent_kv_write(dkv, norm_w, eps: float, pos, inv_freq, rot_dims: int, cache, slots, interleaved: bool = False,
                    amp: float = 1.0):
    """The down-projected K/V row ``dkv [T, rank + rot]``: RMS norm of the latent part, rotary on
    the shared key part (pairs: halves, or neighbours when ``interleaved``; cos and sin times ``amp``),
    both written to the paged cache row ``[rank | rot]`` at ``slots``."""
    if use_native(dkv):
        native_hybrid().latent_kv_write(dkv, norm_w, eps, pos, inv_freq, rot_dims, cache, slots, interleaved, amp)
    else:
        ref.latent_kv_write(dkv, norm_w, eps, pos, inv_freq, rot_dims, cache, slots, interleaved, amp)


def latent_q_assemble(q_lat, q, pos, inv_freq, rot_dims: int, dn: int, interleaved: bool = False, amp: float = 1.0):
    """Query rows in the cache's layout: ``[q_lat | rotary(q[..., dn:])]`` per head, where ``q_lat
    [T, H, rank]`` is the unrotated query part carried into the latent space (q W_uk)."""
    if use_native(q):
        return native_hybrid().latent_q_assemble(q_lat, q, pos, inv_freq, rot_dims, dn, interleaved, amp)
    return ref.latent_q_assemble(q_lat, q, pos, inv_freq, rot_dims, dn, interleaved, amp)


NO_LIMIT = 1 << 30  # a window or chunk that never masks


def latent_attention_prefill(qa, cache, bt, cu, ctx, window: int, sink, scale: float, rk: int, max_q: int,
                             mfma: bool = True, groups: int = 1, koff: int = 0, chunk: int = NO_LIMIT, hscale=None,
                             ofreq=None, sig_bias=None, dist_a=None, dist_b=None, softcap: float = 0.0, keep_first: int = 0):
    """Prompt portions: sequence n's query rows ``[cu[n], cu[n+1])`` end at position ``ctx[n]-1``;
    ``max_q``: the longest portion (sizes the launch).  bf16 shapes that fit run on the matrix cores
    (``mfma=False`` forces the generic fp32-SIMT kernel, which also serves fp32).

    The general form reads a paged row cache whose token rows hold ``groups`` sub-rows (one per kv
    group; query head h reads sub-row ``h // (H // groups)``): entries ``[koff, koff + R)`` of a sub-row
    are the key, its first ``rk`` entries the value.  Latent attention is ``groups=1, koff=0``.  Masks:
    ``window`` (i - j < window) and ``chunk`` (i // chunk == j // chunk), :data:`NO_LIMIT` for none.
    ``sink`` (fp32 [H] or None) joins the softmax denominator; ``hscale`` (fp32 [H]) multiplies a head's
    scores; ``ofreq`` (fp32 [rk/2]) turns the output's neighbour pairs back by ``-position * ofreq``.
    ``dist_a``, ``dist_b`` (fp32 [H], together): ``dist_a ln(1 + dist_b (i - j))`` is taken off the scaled score.
    ``sig_bias`` (fp32 [H]): the weights are not a softmax; a visible key weighs ``sigmoid(score + sig_bias)``
    and nothing is normalised over the keys (no sink then).  ``softcap`` c > 0: the scaled score becomes
    ``c tanh(score / c)`` before masks and softmax; ``keep_first`` n > 0: the window does not hide the keys at
    positions below n (nothing is renumbered: such keys are addressed by their own positions)."""
    if use_native(qa):
        return native_hybrid().latent_attn_prefill(qa, cache, bt, cu, ctx, window, sink, scale, rk, max_q, mfma, groups,
                                                   koff, chunk, hscale, ofreq, sig_bias, dist_a, dist_b, softcap, keep_first)
    return ref.latent_attention(qa, cache, bt, cu, ctx, window, sink, scale, rk, groups, koff, chunk, hscale, ofreq,
                                sig_bias, dist_a, dist_b, softcap, keep_first)


def latent_attention_decode(qa, cache, bt, ctx, window: int, sink, scale: float, rk: int, mfma: bool = True,
                            groups: int = 1, koff: int = 0, chunk: int = NO_LIMIT, hscale=None, ofreq=None,
                            max_ctx: int = 0, sig_bias=None, dist_a=None, dist_b=None, softcap: float = 0.0,
                            keep_first: int = 0):
    """One query row per sequence, at position ``ctx[n] - 1`` (options as in the prefill form;
    ``max_ctx``: the longest context if the host knows it, it sizes the split of the keys)."""
    if use_native(qa):
        return native_hybrid().latent_attn_decode(qa, cache, bt, ctx, window, sink, scale, rk, mfma, groups, koff, chunk,
                                                  hscale, ofreq, max_ctx, sig_bias, dist_a, dist_b, softcap, keep_first)
    cu = torch.arange(qa.shape[0] + 1, dtype=torch.int32)
    return ref.latent_attention(qa, cache, bt, cu, ctx, window, sink, scale, rk, groups, koff, chunk, hscale, ofreq,
                                sig_bias, dist_a, dist_b, softcap, keep_first)


def add_rmsnorm2_f32_(x, a, b, w1, w2, eps: float, one_plus: bool, out_dtype):
    """``x += a (+ b)`` in place on the fp32 residual stream (skipped when ``a`` is None), then RMS norms
    of the same x with weights ``w1`` and (optional) ``w2``: ``x / sqrt(mean(x^2) + eps) * (w + one_plus)``.
    Returns (h1, h2) in ``out_dtype`` (h2 is h1 when ``w2`` is None)."""
    if use_native(x):
        return native_hybrid().add_rmsnorm2_f32_(x, a, b, w1, w2, eps, one_plus, out_dtype == torch.bfloat16)
    return ref.add_rmsnorm2_f32_(x, a, b, w1, w2, eps, one_plus, out_dtype)


def residual_add_act_(x, a, b=None):
    """``x += a (+ b)`` on the fp32 residual stream, a and b in the activation dtype."""
    if use_native(x):
        native_hybrid().residual_add_act_(x, a, b)
        return x
    return ref.residual_add_(x, a, b)


def clamped_glu(gu, limit: float, alpha: float):
    """``gu [T, 2F] = [gate | up]`` -> ``g * sigmoid(alpha g) * (u + 1)`` with ``g = min(gate, limit)``,
    ``u = clamp(up, -limit, limit)``."""
    if use_native(gu):
        return native_hybrid().clamped_glu(gu.contiguous(), limit, alpha)
    return ref.clamped_glu(gu, limit, alpha)


def causal_conv(u, w, state, seq_of, cu, start, sslot, add_input: bool, max_len: int = 0):
    """Short causal convolution over time per channel of the packed rows ``u [T, C]`` (``w`` fp32, tap-major
    ``[taps, C]``): ``y_t = (u_t if add_input) + sum_j w[j] u_(t - taps + 1 + j)``.  ``state`` (fp32
    ``[slots, taps - 1, C]``) carries each live sequence's last ``taps - 1`` inputs between steps (read
    at ``sslot[seq]`` unless the sequence starts at position 0, then updated in place).  ``max_len``: the
    longest portion of the step if the host knows it (steps of short portions take a one-launch form)."""
    if use_native(u):
        return native_hybrid().causal_conv(u, w, state, seq_of, cu, start, sslot, add_input, max_len)
    return ref.causal_conv(u, w, state, seq_of, cu, start, sslot, add_input)


def attn_qkv_prep(z, H: int, G: int, dk: int, dv: int, q_norm, k_norm, eps: float, pos, freq, rot_dims: int,
                  interleaved: bool, amp: float, vfreq, cache, slots, v_from_k: bool = False, v_first=None, v_lambda=None):
    """``z [T, H*dk + G*dk + G*dv] = [q | k | v]``: per-head RMS norm (weights fp32 [dk]; both None: no norm) and
    rotary of q and k, optional turn of v over all of dv by ``position * vfreq``; k and v are written to the
    token's cache row ``[G, dv + dk] = [v | k]`` at ``slots``; returns q ``[T, H, dk]``.  ``v_from_k``: ``z = [q | k]``
    and a token's value is the output of its key projection, taken ahead of norm and rotary (``dv == dk``).  ``v_first`` (``[T, G*dv]``,
    row-strided views allowed) with ``v_lambda`` (fp32, one number): ``v <- (1 - lambda) v + lambda v_first`` before
    the write."""
    if use_native(z):
        return native_hybrid().attn_qkv_prep(z, H, G, dk, dv, q_norm, k_norm, eps, pos, freq, rot_dims, interleaved, amp,
                                             vfreq, cache, slots, v_from_k, v_first, v_lambda)
    return ref.attn_qkv_prep(z, H, G, dk, dv, q_norm, k_norm, eps, pos, freq, rot_dims, interleaved, amp, vfreq, cache, slots,
                             v_from_k, v_first, v_lambda)


def sigmoid_gate_mul(o, g):
    """``o * sigmoid(g)`` -> g's dtype.  ``g`` may have fewer columns than ``o [T, C]``: ``g [T, H]`` gates
    every run of ``C / H`` neighbouring columns (one number per head)."""
    if use_native(g):
        return native_hybrid().sigmoid_gate_mul(o, g)
    return ref.sigmoid_gate_mul(o, g)


MLSTM_CHUNK = 128  # tokens per chunk of the chunk-parallel scan; portions of >= 2 chunks take it


def mlstm_scan(q, k, v, if_raw, b_i, b_f, cap: float, qscale: float, S, n, m, state_slots, cu, start, slab: bool = False,
               cu_host=None):
    """mLSTM recurrence over the step's tokens; returns the un-normalised head outputs fp32
    ``[T, H, dv]`` and updates the state pools in place.  ``slab`` forces the block-per-tile kernel
    (the form for key dims above 128) where the wave-per-tile one would run.  ``cu_host`` (the row
    offsets as a host list) lets long portions run chunk-parallel (:func:`_mlstm_scan_chunked`)."""
    if use_native(q):
        if (cu_host is not None and not slab and q.shape[-1] <= 128
                and max((b - a for a, b in zip(cu_host[:-1], cu_host[1:])), default=0) >= 2 * MLSTM_CHUNK):
            return _mlstm_scan_chunked(q, k, v, if_raw, b_i, b_f, cap, qscale, S, n, m, state_slots, start, cu_host)
        return native_hybrid().mlstm_scan(q, k, v, if_raw, b_i, b_f, cap, qscale, S, n, m, state_slots, cu, start, slab)
    return ref.mlstm_scan(q, k, v, if_raw, b_i, b_f, cap, qscale, S, n, m, state_slots, cu, start)


def _mlstm_scan_chunked(q, k, v, if_raw, b_i, b_f, cap, qscale, S, n, m, state_slots, start, cu_host):
    """The same token-by-token recurrence with the chunks of a portion running side by side.  The state
    is linear in its past: over a chunk with summed log forget gates F and own contribution (S_loc, m_loc)
    -- the chunk run from a zero state with m = -inf -- the carried state becomes m' = max(F + m, m_loc),
    S' = e^(F + m - m') S + e^(m_loc - m') S_loc, and m' is exactly the stabiliser the sequential run
    reaches.  Three passes: (1) every chunk's own contribution, all chunks at once, no outputs; (2) the
    states at every chunk's first token, chunk after chunk (elementwise); (3) every chunk again from its
    true state, all at once, writing the outputs token by token as the sequential form does.  A single
    prompt thus fills chunks x heads x value-tiles waves instead of heads x value-tiles."""
    nat = native_hybrid()
    dev = q.device
    H, dk, dv = q.shape[1], q.shape[2], v.shape[2]
    pcu, base = [0], [0]
    for a, b in zip(cu_host[:-1], cu_host[1:]):
        t = a
        while t < b:
            t = min(t + MLSTM_CHUNK, b)
            pcu.append(t)
        base.append(len(pcu) - 1)
    P = len(pcu) - 1
    i32 = lambda x: torch.tensor(x, dtype=torch.int32).to(dev, non_blocking=True)
    pcu_d, base_d, ident = i32(pcu), i32(base), torch.arange(P, dtype=torch.int32, device=dev)
    f32 = dict(dtype=torch.float32, device=dev)
    locS, locn, locm = torch.empty(P, H, dk, dv, **f32), torch.empty(P, H, dk, **f32), torch.empty(P, H, **f32)
    fsum = torch.empty(P, H, **f32)
    nat.mlstm_scan(q, k, v, if_raw, b_i, b_f, cap, qscale, locS, locn, locm, ident, pcu_d,
                   torch.full((P,), -1, dtype=torch.int32, device=dev), False, fsum, False)
    iS, in_, im = torch.empty_like(locS), torch.empty_like(locn), torch.empty_like(locm)
    nat.mlstm_chunk_combine(S, n, m, state_slots, start, base_d, locS, locn, locm, fsum, iS, in_, im)
    out = nat.mlstm_scan(q, k, v, if_raw, b_i, b_f, cap, qscale, iS, in_, im, ident, pcu_d,
                         torch.ones(P, dtype=torch.int32, device=dev), False, None, True)
    live = [s for s in range(len(base) - 1) if base[s + 1] > base[s]]
    if live:  # the last chunk's final state is the sequence's new carried state
        last = torch.tensor([base[s + 1] - 1 for s in live], dtype=torch.long).to(dev, non_blocking=True)
        dst = state_slots.long()[torch.tensor(live, dtype=torch.long).to(dev, non_blocking=True)]
        S.index_copy_(0, dst, iS.index_select(0, last))
        n.index_copy_(0, dst, in_.index_select(0, last))
        m.index_copy_(0, dst, im.index_select(0, last))
    return out


def headnorm_gate(o, w, g, eps: float, out_dtype, silu: bool = False):
    """Per-head unit-RMS of ``o [T, H, dv]`` (fp32), times ``w [H*dv]`` (None: no weight), times ``sigmoid(g)``
    (``silu``: times ``g sigmoid(g)``)."""
    if use_native(o):
        return native_hybrid().headnorm_gate(o, w, g, eps, out_dtype == torch.bfloat16, silu)
    return ref.headnorm_gate(o, w, g, eps, out_dtype, silu)


def group_topk_router(logits, top: int, groups: int, keep: int):
    """Sigmoid scores of ``logits [T, E]`` (fp32); experts in ``groups`` equal groups of neighbours,
    a group scored by the sum of its two best experts, the ``top`` best experts of the ``keep`` best
    groups chosen.  Returns (expert ids int64 [T, top], their scores fp32 [T, top])."""
    if use_native(logits):
        return native_hybrid().group_topk_router(logits, top, groups, keep)
    return ref.group_topk_router(logits, top, groups, keep)


def swiglu_any(gu):
    """``silu(gate) * up`` of ``gu [..., 2F]`` = ``[gate | up]``, bf16 or fp32."""
    return glu_act(gu, "silu")


def glu_act(gu, kind: str, scale=None):
    """``act(gate) * up`` of ``gu [rows, 2F]`` = ``[gate | up]`` (row-strided views allowed), bf16 or fp32, computed
    in fp32; ``kind``: ``silu`` or ``gelu_tanh`` (the tanh form of the GELU); ``scale`` (fp32 ``[rows]``): a factor
    per row."""
    if use_native(gu):
        return native_hybrid().glu_act(gu, {"silu": 0, "gelu_tanh": 1}[kind], scale)
    return ref.glu_act(gu, kind, scale)


def gated_norm_add_norm_f32_(x, y, r, w_post, w_next, eps: float, out_dtype):
    """A sublayer's result into the fp32 residual stream of a layer with norms on both sides and a
    gated residual, in one pass: ``g = y sigmoid(r)``; ``x += g / rms(g) * w_post`` in place; returns
    ``x / rms(x) * w_next`` -> ``out_dtype`` (the next sublayer's input), or None when ``w_next`` is None.
    ``y`` and ``r`` are ``[T, W]`` in the activation dtype or fp32 (row-strided views allowed)."""
    if use_native(x):
        h = native_hybrid().gated_norm_add_norm_f32_(x, y, r, w_post, w_next, eps, out_dtype == torch.bfloat16)
        return h if w_next is not None else None
    return ref.gated_norm_add_norm_f32_(x, y, r, w_post, w_next, eps, out_dtype)


def embed_rmsnorm_f32(ids, pos, table, pos_table, w, eps: float, out_dtype):
    """``x = table[ids] + pos_table[pos]`` (learned absolute positions) as the fp32 residual stream, and
    its RMS norm with weight ``w`` -> ``out_dtype``.  Returns (x, h)."""
    if use_native(table):
        return native_hybrid().embed_rmsnorm_f32(ids, pos, table, pos_table, w, eps, out_dtype == torch.bfloat16)
    return ref.embed_rmsnorm_f32(ids, pos, table, pos_table, w, eps, out_dtype)


GLA_CHUNK = 64  # tokens per chunk of the chunk-parallel scan; portions of >= 4 chunks take it


def gla_chunk_plan(cu_host, device):
    """The chunks of a step's portions for the chunk-parallel scan, or None when no portion is long enough:
    (chunk row offsets, first chunk of every sequence, 0 .. P-1, P zeros, P ones) on ``device`` and P.  It
    depends on the step only, so the layers of a model share one."""
    if cu_host is None or max((b - a for a, b in zip(cu_host[:-1], cu_host[1:])), default=0) < 4 * GLA_CHUNK:
        return None
    pcu, base = [0], [0]
    for a, b in zip(cu_host[:-1], cu_host[1:]):
        t = a
        while t < b:
            t = min(t + GLA_CHUNK, b)
            pcu.append(t)
        base.append(len(pcu) - 1)
    P = len(pcu) - 1
    both = torch.tensor(pcu + base, dtype=torch.int32).to(device)  # blocking: the host tensor is a temporary
    ident = torch.arange(P, dtype=torch.int32, device=device)
    return (both[:P + 1], both[P + 1:], ident, torch.zeros(P, dtype=torch.int32, device=device),
            torch.ones(P, dtype=torch.int32, device=device), P)


def gla_scan(q, k, v, z, z_bias, tau: float, qscale: float, S, state_slots, cu, start, cu_host=None, plan=None):
    """Gated linear attention over the step's tokens: per head a memory ``S [dk, dv]`` with a decay per
    key channel, ``a_t = sigmoid(z_t + z_bias)^(1/tau)`` (computed as ``exp(log_sigmoid / tau)`` in fp32),
    ``S_t = diag(a_t) S_(t-1) + k_t v_t^T``, ``o_t = S_t^T (q_t qscale)``.  ``q, k [T, H, dk]``, ``v [T, H, dv]``
    (row-strided views allowed), ``z [T, H*dk]`` fp32, ``z_bias`` fp32 ``[H*dk]``.
    Returns fp32 ``[T, H, dv]`` and updates the state pool ``S [slots, H, dk, dv]`` in place at
    ``state_slots[seq]`` (a sequence with ``start == 0`` begins from zeros).  ``cu_host`` (the row offsets on
    the host) or ``plan`` (:func:`gla_chunk_plan` of them) lets long portions run chunk-parallel."""
    if use_native(q):
        nat = native_hybrid()
        if plan is None and cu_host is not None:
            plan = gla_chunk_plan(cu_host, q.device)
        if plan is not None:
            return _gla_scan_chunked(nat, q, k, v, z, z_bias, tau, qscale, S, state_slots, start, plan)
        return nat.gla_scan(q, k, v, z, z_bias, tau, qscale, S, state_slots, cu, start, None, True, True)
    return ref.gla_scan(q, k, v, z, z_bias, tau, qscale, S, state_slots, cu, start)


def _gla_scan_chunked(nat, q, k, v, z, z_bias, tau, qscale, S, state_slots, start, plan):
    """The same recurrence with the chunks of a portion side by side.  The memory is linear in its past:
    over a chunk with total decay D (the product of its a_t per key channel) and own contribution S_loc (the
    chunk run from zeros), S_end = diag(D) S_begin + S_loc.  Three passes: (1) every chunk from zeros, all at
    once, no outputs, giving (S_loc, log D); (2) the memory at every chunk's first token, chunk after chunk
    (elementwise), and the sequence's new carried memory; (3) every chunk again from its true memory, all at
    once, writing outputs token by token."""
    pcu_d, base_d, ident, zeros, ones, P = plan
    H, dk, dv = q.shape[1], q.shape[2], v.shape[2]
    f32 = dict(dtype=torch.float32, device=q.device)
    loc, logd = torch.empty(P, H, dk, dv, **f32), torch.empty(P, H, dk, **f32)
    nat.gla_scan(q, k, v, z, z_bias, tau, qscale, loc, ident, pcu_d, zeros, logd, False, True)
    init = torch.empty_like(loc)
    nat.gla_chunk_combine(S, state_slots, start, base_d, loc, logd, init)
    return nat.gla_scan(q, k, v, z, z_bias, tau, qscale, init, ident, pcu_d, ones, None, True, False)


def qk_fullnorm_prep(z, H: int, G: int, dk: int, dv: int, q_norm, k_norm, eps: float, pos, temp_coef: float,
                     temp_every: int, cache, slots, freq=None, rot_dims: int = 0, interleaved: bool = False, amp: float = 1.0):
    """``z [T, >= H*dk + G*dk + G*dv] = [q | k | v | ...]`` (biases already added): RMS norm over the whole
    of q and over the whole of k before the split into heads (weights fp32 ``[H*dk]``, ``[G*dk]``); the query
    temperature ``1 + temp_coef ln(floor((p + 1) / temp_every) + 1)`` at position p (``temp_coef`` 0: none); rotary of
    q and k on the first ``rot_dims`` entries of every head (0: none; pairs are neighbours or halves, ``freq`` fp32
    ``[rot_dims / 2]``, cos and sin times ``amp``); k and v are written to the token's cache row ``[G, dv + dk] = [v | k]``
    at ``slots``; returns q ``[T, H, dk]``."""
    a = (z, H, G, dk, dv, q_norm, k_norm, eps, pos, temp_coef, temp_every, cache, slots, freq if rot_dims else None, rot_dims,
         interleaved, amp)
    return native_hybrid().qk_fullnorm_prep(*a) if use_native(z) else ref.qk_fullnorm_prep(*a)


def bias_topk_router(logits, bias, top: int, groups: int = 1, keep: int = 1, renorm: bool = True):
    """Softmax scores of ``logits [T, E]`` (fp32); the ``top`` experts with the largest ``score + bias`` (the
    choice score; ``bias`` None: the score) are chosen (ties: the lower index).  ``groups`` > 1: the experts
    form that many equal groups of neighbours, a group's score is its largest choice score, and only experts
    of the ``keep`` best groups can be chosen.  The weights are the chosen experts' own scores (without the
    bias), over their sum (+ 1e-20) when ``renorm``.  Returns (expert ids int64 [T, top], weights fp32 [T, top])."""
    if use_native(logits):
        return native_hybrid().bias_topk_router(logits, bias, top, groups, keep, renorm)
    return ref.bias_topk_router(logits, bias, top, groups, keep, renorm)


def act_any(x, kind: str, scale=None):
    """Elementwise activation of ``x`` (bf16 or fp32, computed in fp32): ``relu2`` = relu(x)^2, ``gelu`` = the
    exact (erf) GELU; ``scale`` (fp32 ``[rows]``): a factor per row."""
    if use_native(x):
        return native_hybrid().act_any(x, {"relu2": 0, "gelu": 1}[kind], scale)
    return ref.act_any(x, kind, scale)


def hc_embed_norm(ids, table, streams: int, c_in, g, eps: float, out_dtype):
    """The start of ``streams`` residual streams (hyper-connections): every stream is the embedding row.
    Returns (``X`` fp32 ``[T, streams, W]``, the first sublayer's input ``norm(sum_s c_in[s] x_s) * g`` ->
    ``out_dtype``); ``c_in`` fp32 ``[streams]``, ``g`` fp32, one number (an RMS norm with a single weight)."""
    if use_native(table):
        return native_hybrid().hc_embed_norm(ids, table, streams, c_in, g, eps, out_dtype == torch.bfloat16)
    return ref.hc_embed_norm(ids, table, streams, c_in, g, eps, out_dtype)


def hc_update_norm_(X, y1, s1: float, y2, s2: float, mix, c_out, mult: float, c_in, g, eps: float, out_dtype):
    """A sublayer's result into the residual streams ``X`` (fp32 ``[T, S, W]``, in place), all streams at once
    from the old ones: ``x_t <- sum_s mix[s, t] x_s + mult c_out[t] (s1 y1 + s2 y2)`` (``y2`` may be None; ``y``
    ``[T, W]`` in the activation dtype or fp32, row-strided views allowed), and the next sublayer's input
    ``norm(sum_t c_in[t] x_t) * g`` -> ``out_dtype`` in the same pass over the row (None when ``c_in`` is None).
    One stream with ``mix = c_out = c_in = 1`` is the plain residual sum with a pre-norm."""
    if use_native(X):
        h = native_hybrid().hc_update_norm_(X, y1, s1, y2, s2, mix, c_out, mult, c_in, g, eps, out_dtype == torch.bfloat16)
        return h if c_in is not None else None
    return ref.hc_update_norm_(X, y1, s1, y2, s2, mix, c_out, mult, c_in, g, eps, out_dtype)


def delta_scan(r, k, v, zw, w0, za, ab, decay_coef: float, key_eps: float, S, state_slots, cu, start, cu_host=None, plan=None):
    """The generalized delta rule over the step's tokens: per head a memory ``S [dk, dv]``; with the decay
    ``w = exp(-decay_coef sigmoid(zw + w0))`` and the removal rate ``a = sigmoid(za + ab)`` per key channel and the
    unit key ``u = k / sqrt(sum k^2 + key_eps)``, ``S_t = diag(w_t) S_(t-1) - (a_t u_t) (u_t^T S_(t-1)) + k_t v_t^T``
    (both terms read the old memory) and ``o_t = S_t^T r_t``.  ``r, k [T, H, dk]``, ``v [T, H, dv]`` (row-strided
    views allowed), ``zw`` fp32 ``[T, H*dk]``, ``za [T, H*dk]`` (any float dtype), ``w0``, ``ab`` fp32 ``[H*dk]``.
    Returns fp32 ``[T, H, dv]`` and updates the state pool ``S [slots, H, dk, dv]`` in place at ``state_slots[seq]``
    (a sequence with ``start == 0`` begins from zeros).  ``plan`` (:func:`gla_chunk_plan` of the row offsets)
    lets long portions run chunk-parallel."""
    if use_native(r):
        nat = native_hybrid()
        if plan is None and cu_host is not None:
            plan = gla_chunk_plan(cu_host, r.device)
        if plan is not None and DELTA_CHUNKED and _delta_combine_fits(k.shape[2], v.shape[2]):
            return _delta_scan_chunked(nat, r, k, v, zw, w0, za, ab, decay_coef, key_eps, S, state_slots, start, plan)
        return nat.delta_scan(r, k, v, zw, w0, za, ab, decay_coef, key_eps, S, state_slots, cu, start, None, True, True)
    return ref.delta_scan(r, k, v, zw, w0, za, ab, decay_coef, key_eps, S, state_slots, cu, start)


DELTA_CHUNKED = True  # long portions run chunk-parallel


def _delta_combine_fits(dk: int, dv: int) -> bool:
    """The combine pass holds a head's memory and a chunk's transition product in LDS and tiles them 4 x 4."""
    return dk % 4 == 0 and dv % 4 == 0 and 4 * dk * (dk + dv) <= 65536 and dk * dk <= 48 * 256 and dk * dv <= 8192


def _delta_scan_chunked(nat, r, k, v, zw, w0, za, ab, decay_coef, key_eps, S, state_slots, start, plan):
    """The same recurrence with the chunks of a portion side by side.  The memory is linear in its past: a token
    maps it by ``A_t = diag(w_t) - (a_t u_t) u_t^T`` and adds ``k_t v_t^T``, so over a chunk with transition product
    ``P = A_n ... A_1`` and own contribution ``S_loc`` (the chunk run from zeros), ``S_end = P S_begin + S_loc``.  Three
    passes: (1) every chunk from zeros and, in further waves of the same launch, from the identity without the
    ``k v^T`` term, all at once, no outputs, giving ``(S_loc, P^T)``; (2) the memory at every chunk's first token, chunk
    after chunk, and the sequence's new carried memory; (3) every chunk again from its true memory, all at once,
    writing outputs token by token."""
    pcu_d, base_d, ident, zeros, ones, Pn = plan
    H, dk, dv = r.shape[1], r.shape[2], v.shape[2]
    f32 = dict(dtype=torch.float32, device=r.device)
    loc, prod = torch.empty(Pn, H, dk, dv, **f32), torch.empty(Pn, H, dk, dk, **f32)
    nat.delta_scan(r, k, v, zw, w0, za, ab, decay_coef, key_eps, loc, ident, pcu_d, zeros, prod, False, True)
    init = torch.empty_like(loc)
    nat.delta_chunk_combine(S, state_slots, start, base_d, loc, prod, init)
    return nat.delta_scan(r, k, v, zw, w0, za, ab, decay_coef, key_eps, init, ident, pcu_d, ones, None, True, False)


def tanh_act(x):
    """Elementwise ``tanh`` (computed in fp32) -> x's dtype."""
    if use_native(x):
        return native_hybrid().tanh_act(x.contiguous())
    return ref.tanh_act(x)


def softcap_(x, cap: float):
    """``x <- cap tanh(x / cap)`` in place on an fp32 tensor."""
    if use_native(x):
        native_hybrid().softcap_(x, cap)
        return x
    return ref.softcap_(x, cap)



def gated_add_f32_(out, y, g):
    """``out += y * sigmoid(g)`` in place on the fp32 ``out [T, W]``; ``y [T, W]`` in any float dtype, ``g [T, 1]``
    one gate logit per row (row-strided views allowed)."""
    if use_native(out):
        native_hybrid().gated_add_f32_(out, y, g)
        return out
    return ref.gated_add_f32_(out, y, g)


def _norm_conv_fits(W: int, groups: int, taps: int) -> bool:
    """The one-pass form: 2 to 4 taps, groups of whole column quads, rows up to 8192 wide."""
    return 2 <= taps <= 4 and W % groups == 0 and (W // groups) % 4 == 0 and W <= 8192


def _conv_of_normed(h, cw, state, b, out_dtype):
    """``h + conv(h)`` of an fp32 h (the second half of the unfused form)."""
    return causal_conv(h, cw, state, b.seq_of, b.cu, b.start, b.state, True, max_len=max(b.max_q, 1 if h.shape[0] > b.Tp else 0)).to(out_dtype)


def group_norm_f32(x, y, w, groups: int, eps: float, out_dtype):
    """``x + y`` (``y`` None: x) of the fp32 residual stream ``[T, W]``, and its RMS norm in ``groups`` equal
    consecutive parts, each over its own root mean square, the whole times ``w [W]`` -> ``out_dtype``."""
    if use_native(x):
        xo, h = native_hybrid().group_norm_f32(x, y, w, groups, eps, out_dtype == torch.bfloat16)
        return (xo if y is not None else x), h
    return ref.group_norm_f32(x, y, w, groups, eps, out_dtype)


def add_norm_conv(x, y, w, groups: int, eps: float, cw, state, b, out_dtype):
    """A sublayer's result into the fp32 residual stream and the next sublayer's input in one pass:
    ``x <- x + y``; ``h = norm(x)`` in ``groups`` equal parts (:func:`group_norm_f32`); the result is ``h_t + sum_j cw[j]
    h_(t - taps + 1 + j)`` per sequence and channel (``cw`` fp32, tap-major ``[taps, W]``) -> ``out_dtype``.
    ``state`` (fp32 ``[slots, taps - 1, W]``) carries the last ``taps - 1`` rows of h of every live sequence between
    steps; h is not rounded before the convolution.  ``b``: the step (:class:`~llmctl.models.mixers.StepBatch`).
    Returns (the new stream, the input); ``x`` itself is left as it was."""
    if use_native(x):
        if _norm_conv_fits(x.shape[1], groups, cw.shape[0]):
            return native_hybrid().add_norm_conv(x, y, w, groups, eps, cw, state, b.seq_of, b.cu, b.start, b.state,
                                                 b.carried, out_dtype == torch.bfloat16)
        x, h = group_norm_f32(x, y, w, groups, eps, torch.float32)
        return x, _conv_of_normed(h, cw, state, b, out_dtype)
    x, h = ref.group_norm_f32(x, y, w, groups, eps, torch.float32)
    return x, ref.causal_conv(h, cw, state, b.seq_of, b.cu, b.start, b.state, True).to(out_dtype)


def embed_norm_conv(table, pos_table, scale: float, w, groups: int, eps: float, cw, state, b):
    """The start of the stream, ``x = table[id] * scale + pos_table[position]`` (fp32), and the first sublayer's input
    as in :func:`add_norm_conv` (in the tables' dtype).  Returns (x, input)."""
    if use_native(table):
        if _norm_conv_fits(table.shape[1], groups, cw.shape[0]):
            return native_hybrid().embed_norm_conv(b.ids, b.pos, table, pos_table, scale, w, groups, eps, cw, state,
                                                   b.seq_of, b.cu, b.start, b.state, b.carried)
        x = table[b.ids].float() * scale + pos_table[b.pos.long()].float()
        _, h = group_norm_f32(x, None, w, groups, eps, torch.float32)
        return x, _conv_of_normed(h, cw, state, b, table.dtype)
    x = table[b.ids].float() * scale + pos_table[b.pos.long()].float()
    _, h = ref.group_norm_f32(x, None, w, groups, eps, torch.float32)
    return x, ref.causal_conv(h, cw, state, b.seq_of, b.cu, b.start, b.state, True).to(table.dtype)


MINGRU_CHUNK = 32  # tokens per chunk of the chunk-parallel scan; portions of >= 2 chunks take it
MINGRU_MAX_CHUNKS = 128  # longer portions get longer chunks


def mingru_scan(z, z_bias, x_bias, S, b, chunk: int = 0):
    """The minGRU recurrence over the step's tokens with its output gate: rows ``z [T, >= 3 W]`` = ``[z | x | g]``,
    ``zeta = sigmoid(z + z_bias)``, ``u = x + x_bias``, ``cand = u + 1/2`` where ``u >= 0`` and ``sigmoid(u)`` elsewhere,
    ``S_t = (1 - zeta) S_(t-1) + zeta cand``; returns ``S_t silu(g)`` ``[T, W]`` in z's dtype.  Everything is fp32 inside;
    the pool ``S`` (fp32 ``[slots, W]``) is updated in place at ``b.state`` (a sequence that starts at position 0
    begins from zeros).  Long portions run in chunks side by side: a chunk maps the state by ``S -> A S + B`` per
    channel, so a first pass forms every chunk's (A, B) and a second one folds those before it and writes the outputs.
    ``chunk`` > 0 fixes the chunk length."""
    if use_native(z):
        portions = b.p_ctx.shape[0] if b.p_ctx is not None else 0
        if not chunk:
            chunk = MINGRU_CHUNK
            while chunk * MINGRU_MAX_CHUNKS < b.max_q:
                chunk *= 2
        return native_hybrid().mingru_scan(z, z_bias, x_bias, S, b.state, b.cu, b.start, portions, b.max_q, chunk)
    return ref.mingru_scan(z, z_bias, x_bias, S, b.state, b.cu, b.start)


def kv_rows_write(k, v, cache, slots, groups: int):
    """Keys ``k [T, groups * kw]`` and values ``v [T, groups * vw]`` (column views allowed) to the tokens' cache rows
    ``[groups, vw + kw] = [v | k]`` at ``slots``."""
    if use_native(k):
        native_hybrid().kv_rows_write(k, v, cache, slots, groups)
    else:
        ref.kv_rows_write(k, v, cache, slots, groups)


def diff_attention(q, cache, bt, cu, ctx, heads: int, groups: int, dk: int, dv: int, window: int, scale: float, lam,
                   post: float, eps: float, out, max_q: int = 1, max_ctx: int = 0, mfma: bool = True):
    """Differential attention over a paged row cache.  A token's row holds ``groups`` sub-rows ``[v (dv) | k_1 (dk) |
    k_2 (dk)]``; query rows are ``[heads, 2, dk]`` (the first columns of ``q``, row-strided views allowed) and head h
    reads sub-row ``h // (heads // groups)``.  Map m is an ordinary softmax attention of scores ``q_m . k_m * scale`` over the
    keys inside the causal ``window`` (i - j < window; :data:`NO_LIMIT`: plain causal); with the maps' outputs ``a_1, a_2``
    a head gives ``o = a_1 - lam a_2`` (``lam``: fp32, one number), then ``post * o / sqrt(mean(o^2) + eps)`` over its dv
    values, written to ``out [rows, heads * dv]``.  ``cu`` given: portions, sequence n's rows ``[cu[n], cu[n+1])`` end at
    position ``ctx[n] - 1`` and the longest has ``max_q``; ``cu`` None: one row per sequence at ``ctx[n] - 1`` (``max_ctx``:
    the longest context if the host knows it).  ``mfma=False`` forces the generic fp32-SIMT kernel, which also serves
    fp32 and shapes that do not fit the matrix cores."""
    if use_native(q):
        native_hybrid().diff_attn(q, cache, bt, cu, ctx, heads, groups, dk, dv, window, scale, lam, post, eps, max_q, max_ctx,
                                  mfma, out)
    else:
        ref.diff_attention(q, cache, bt, cu, ctx, heads, groups, dk, dv, window, scale, lam, post, eps, out)
    return out


def conv_silu_unit(u, w, bias, state, b, nq: int, nk: int, dk: int, qscale: float, eps: float = 1e-6):
    """Short causal convolutions over time with silu, ``silu(sum_j w[j] u_(t - taps + 1 + j) + bias)`` per channel of the packed
    rows ``u [T, C]`` (``w`` fp32, tap-major ``[taps, C]``; ``bias`` fp32 ``[C]`` or None), for the inputs of a recurrence:
    the first ``nq`` groups of ``dk`` channels, then ``nk`` more, become unit vectors ``x / sqrt(sum x^2 + eps)`` (the first
    ones times ``qscale``).  ``state`` (fp32 ``[slots, taps - 1, C]``) carries each live sequence's last ``taps - 1`` inputs.
    Returns (unit vectors fp32 ``[T, nq + nk, dk]`` or None, the other channels ``[T, C - (nq + nk) dk]`` in u's dtype)."""
    if use_native(u):
        qk, y = native_hybrid().conv_silu_unit(u, w, bias, state, b.seq_of, b.cu, b.start, b.state, nq, nk, dk, qscale, eps,
                                               max(b.max_q, 1 if u.shape[0] > b.Tp else 0))
        return (qk if nq + nk else None), y
    return ref.conv_silu_unit(u, w, bias, state, b.cu, b.start, b.state, nq, nk, dk, qscale, eps)


def rotary_f32(z, nq: int, nk: int, dk: int, pos, freq, rot_dims: int, interleaved: bool, amp: float = 1.0, kscale: float = 1.0):
    """Rotary of the heads ``z [T, >= (nq + nk) dk]`` (``nq`` query heads, then ``nk`` key heads; pairs are halves, or
    neighbours when ``interleaved``) for a recurrence: fp32 ``[T, nq + nk, dk]``, keys times ``kscale`` after the turn."""
    a = (z, nq, nk, dk, pos, freq, rot_dims, interleaved, amp, kscale)
    return native_hybrid().rotary_f32(*a) if use_native(z) else ref.rotary_f32(*a)


MEMORY_CHUNK = 64  # tokens per chunk of a memory scan
MEMORY_KINDS = {"fixed": 0, "ssm": 1, "delta": 2}


def _memory_plan(b, device):
    """The chunks of a step's prompt portions when one of them is longer than a chunk, else None: (chunk row offsets, first
    chunk of every portion) on ``device`` and the number of chunks.  It depends on the step only; layers share it."""
    if "memory_plan" not in b.scratch:
        plan = None
        if b.max_q > MEMORY_CHUNK:
            n = b.p_ctx.shape[0]
            pcu, base = [0], [0]
            for lo, hi in zip(b.cu_host[:n], b.cu_host[1:n + 1]):
                pcu += list(range(lo + MEMORY_CHUNK, hi, MEMORY_CHUNK)) + ([hi] if hi > lo else [])
                base.append(len(pcu) - 1)
            both = torch.tensor(pcu + base, dtype=torch.int32).to(device)  # blocking: the host tensor is a temporary
            plan = (both[:len(pcu)], both[len(pcu):], len(pcu) - 1)
        b.scratch["memory_plan"] = plan
    return b.scratch["memory_plan"]


def memory_scan(q, k, v, kind: str, S, b, ga=None, gb=None, a_log=None, dt_bias=None, log_decay=None, skip=None, norm=None):
    """A matrix memory per head with one decay per head and token, over the step's tokens: ``S_t = g_t S_(t-1) + k_t u_t^T``, ``o_t =
    S_t^T q_t`` with ``u_t = beta_t v_t``, or ``u_t = beta_t (v_t - g_t S_(t-1)^T k_t)`` (what the decayed memory gives for k is
    taken off first).

    ``kind`` says where g and beta come from (fp32 here): ``fixed``: ``g = exp(log_decay_h)``, beta = 1; ``ssm``: ``beta = dt =
    softplus(ga + dt_bias)``, ``g = exp(-exp(a_log) dt)``; ``delta``: g likewise, ``beta = sigmoid(gb)`` and the subtracting
    form of u.  ``q, k [T, KH, dk]`` (one dtype; head h of H reads h // (H / KH)), ``v [T, H, dv]`` (row-strided views
    allowed), ``ga, gb [T, H]`` in v's dtype, ``a_log, dt_bias, log_decay, skip`` fp32 ``[H]``; ``skip``: o gains ``skip_h v``.
    Returns fp32 ``[T, H, dv]`` and updates the state pool ``S`` (fp32 ``[slots, H, dk, dv]``) in place at ``b.state`` (a
    sequence that starts at position 0 begins from zeros).  ``norm`` = (weight fp32 ``[H*dv]`` or None, gate ``[T, H*dv]``, eps):
    returns :func:`headnorm_gate` of the outputs with silu, ``[T, H*dv]`` in v's dtype (in the same kernels for value sizes
    up to 128 in quads).

    Decode rows run one after the other in memory (a read and a write of S); prompt portions run in chunks of
    :data:`MEMORY_CHUNK` tokens whose products go to the fp32 matrix cores.  A portion of several chunks takes three
    passes: every chunk's own contribution (delta: and its transition product) at once, the memories at the
    chunks' first tokens in order, every chunk's outputs at once."""
    if not use_native(v):
        o = ref.memory_scan(q, k, v, kind, ga, gb, a_log, dt_bias, log_decay, skip, S, b.state, b.cu, b.start)
        return o if norm is None else ref.headnorm_gate(o, norm[0], norm[1], norm[2], v.dtype, True)
    nat = native_hybrid()
    T, H, dv = v.shape
    dk = q.shape[2]
    if norm is not None and (dv % 4 or dv > 128):
        o = memory_scan(q, k, v, kind, S, b, ga, gb, a_log, dt_bias, log_decay, skip)
        return headnorm_gate(o, *norm, v.dtype, True)
    if norm is None:
        out, ends = torch.empty(T, H, dv, device=v.device, dtype=torch.float32), (None, None, 0.0)
    else:
        out, ends = torch.empty(T, H * dv, device=v.device, dtype=v.dtype), norm
    gates = (MEMORY_KINDS[kind], ga, gb, a_log, dt_bias, log_decay, skip)
    if b.Tp:
        n = b.p_ctx.shape[0]
        plan = _memory_plan(b, v.device)
        if plan is None:
            nat.memory_chunks(q, k, v, *gates, S, b.state[:n], b.cu[:n + 1], b.start[:n], None, out, *ends, b.Tp)
        else:
            pcu, base, P = plan
            f32 = dict(dtype=torch.float32, device=v.device)
            loc = torch.empty(P, H, dk, dv, **f32)
            dec = torch.empty(P, H, **f32)
            dkp = (dk + 15) // 16 * 16
            trans = torch.empty(P, H, dkp, dkp, **f32) if kind == "delta" else None
            init = torch.empty(P, H, dk, dv, **f32)
            nat.memory_chunk_local(q, k, v, *gates, pcu, loc, dec, trans)
            nat.memory_combine(S, b.state[:n], b.start[:n], base, loc, dec, trans, init)
            nat.memory_chunks(q, k, v, *gates, S, None, pcu, None, init, out, *ends, b.Tp)
    if T > b.Tp:
        n0 = b.cu.shape[0] - 1 - (T - b.Tp)
        nat.memory_decode(q, k, v, *gates, S, b.state[n0:], b.start[n0:], out, *ends, b.Tp)
    return out


def gate_groupnorm(o, z, w, groups: int, eps: float, out_dtype):
    """``y = o silu(z)`` (o fp32 ``[T, C]``, z ``[T, C]``), then an RMS norm of y in ``groups`` equal consecutive parts, each
    over its own root mean square, the whole times ``w [C]``."""
    if use_native(o):
        return native_hybrid().gate_groupnorm(o, z, w, groups, eps, out_dtype == torch.bfloat16)
    return ref.gate_groupnorm(o, z, w, groups, eps, out_dtype)


def norm_add_f32_(x, y1, s1: float, y2, s2: float, w, mult: float, eps: float, one_plus: bool, out_dtype):
    """The end of a sublayer whose only norm is on its result: ``y = s1 y1 (+ s2 y2)``, ``x += mult y / rms(y) (w + one_plus)``
    in place on the fp32 stream, and the next sublayer's input, x itself, in ``out_dtype``.  ``y [T, W]`` in the activation
    dtype (row-strided views allowed)."""
    if use_native(x):
        return native_hybrid().norm_add_f32_(x, y1, s1, y2, s2, w, mult, eps, one_plus, out_dtype == torch.bfloat16)
    return ref.norm_add_f32_(x, y1, s1, y2, s2, w, mult, eps, one_plus, out_dtype)


def embed_f32(ids, table):
    """The embedding rows as the fp32 residual stream and in the table's dtype: (x, h)."""
    if use_native(table):
        return native_hybrid().embed_f32(ids, table)
    return ref.embed_f32(ids, table)
