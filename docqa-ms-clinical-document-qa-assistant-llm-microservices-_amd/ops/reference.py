"""Plain-PyTorch (fp32-accumulating) reference implementations of every native op.

These serve two purposes:
  * the numerics oracle the GPU tests compare the HIP kernels against;
  * the CPU execution path, so services, models and the distributed code can be
    exercised in CI without a GPU.  On a GPU tensor the dispatcher in
    ``docqa_amd.ops`` never falls back here: it raises if the native extension is
    missing (see ``ops/__init__.py``).
Layouts mirror the kernels exactly (paged cache ``[num_blocks, Hkv, BS, D]``, packed
QKV rows ``[(Hq + 2*Hkv) * D]``, FAISS distance conventions).
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F


def rmsnorm(x, w, eps):
    xf = x.float()
    inv = torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    return (xf * inv * w.float()).to(x.dtype)


def add_rmsnorm(x, residual, w, eps):
    s = (x.float() + residual.float()).to(x.dtype)
    residual.copy_(s)
    return rmsnorm(s, w, eps)


def layernorm(x, residual, gamma, beta, eps):
    xf = x.float()
    if residual is not None:
        xf = xf + residual.float()
    return F.layer_norm(xf, (x.shape[-1],), gamma.float(), beta.float(), eps).to(x.dtype)


def rope_inv_freq(head_dim: int, theta: float, scaling: dict | None = None) -> torch.Tensor:
    """fp64 RoPE inverse frequencies, with Hugging Face ``rope_scaling`` applied.

    * ``None`` / ``"default"``: theta^(-2i/d).
    * ``"linear"``: every frequency divided by ``factor`` (position interpolation).
    * ``"llama3"`` (Llama-3.1 / 3.2): wavelengths longer than
      ``original_max_position_embeddings / low_freq_factor`` are divided by ``factor``,
      shorter than ``.../high_freq_factor`` kept, and the band between is blended with
      ``s = (L_orig / wavelen - low) / (high - low)``: ``(1 - s) * f / factor + s * f``.
    Anything else raises: a checkpoint must not load with silently wrong positions."""
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    if not scaling:
        return inv
    kind = scaling.get("rope_type", scaling.get("type", "default"))
    if kind == "default":
        return inv
    factor = float(scaling["factor"])
    if kind == "linear":
        return inv / factor
    if kind == "llama3":
        low, high = float(scaling["low_freq_factor"]), float(scaling["high_freq_factor"])
        orig = float(scaling["original_max_position_embeddings"])
        wavelen = 2 * math.pi / inv
        scaled = torch.where(wavelen > orig / low, inv / factor, inv)
        smooth = (orig / wavelen - low) / (high - low)
        blended = (1 - smooth) * scaled / factor + smooth * scaled
        medium = (wavelen >= orig / high) & (wavelen <= orig / low)
        return torch.where(medium, blended, scaled)
    raise NotImplementedError(f"rope_scaling type {kind!r} is not supported")


def rope_cos_sin(max_pos: int, head_dim: int, theta: float, device=None,
                 scaling: dict | None = None) -> torch.Tensor:
    """fp32 table [max_pos, head_dim]: first half cos, second half sin (rotate-half RoPE)."""
    inv_freq = rope_inv_freq(head_dim, theta, scaling)
    t = torch.arange(max_pos, dtype=torch.float64)
    freqs = torch.outer(t, inv_freq)
    return torch.cat([freqs.cos(), freqs.sin()], dim=-1).float().to(device)


def rope_cache(qkv, positions, cos_sin, slot_mapping, k_cache, v_cache, Hq, Hkv, D):
    T = qkv.shape[0]
    x = qkv.view(T, Hq + 2 * Hkv, D)
    cs = cos_sin[positions.long()]  # [T, D]
    half = D // 2
    cos, sin = cs[:, None, :half], cs[:, None, half:]
    qk = x[:, : Hq + Hkv].float()
    x1, x2 = qk[..., :half], qk[..., half:]
    rot = torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1).to(qkv.dtype)
    x[:, : Hq + Hkv] = rot
    if slot_mapping is not None:
        BS = k_cache.shape[2]
        sm = slot_mapping.long()
        valid = sm >= 0
        sm = sm[valid]
        blk, off = sm // BS, sm % BS
        k = x[valid, Hq : Hq + Hkv]
        v = x[valid, Hq + Hkv :]
        k_cache[blk, :, off] = k
        v_cache[blk, :, off] = v


def silu_mul(gu, interleaved: bool = False):
    """SwiGLU; ``interleaved``: gate|up rows in blocks of 8 (glu_interleave layout)."""
    if interleaved:
        v = gu.float().unflatten(-1, (-1, 2, 8))
        g, u = v[..., 0, :].flatten(-2), v[..., 1, :].flatten(-2)
    else:
        g, u = gu.float().chunk(2, dim=-1)
    return (F.silu(g) * u).to(gu.dtype)


def glu_interleave(gate, up):
    """[I, K] gate and up -> [2I, K] with rows in blocks of 8: g0..g7 u0..u7 g8..g15 ..."""
    I, K = gate.shape
    return torch.stack([gate.view(I // 8, 8, K), up.view(I // 8, 8, K)], 1).reshape(2 * I, K)


def glu_split(gu):
    """Inverse of :func:`glu_interleave`."""
    v = gu.view(-1, 2, 8, gu.shape[-1])
    return v[:, 0].reshape(-1, gu.shape[-1]), v[:, 1].reshape(-1, gu.shape[-1])


def bias_act(x, bias, residual, gelu):
    y = x.float()
    if residual is not None:
        y = y + residual.float()
    y = y + bias.float()
    if gelu:
        y = F.gelu(y)  # erf form
    return y.to(x.dtype)


def linear_fused(x, w, bias, residual, epi):
    """epi: 0 none, 1 bias, 2 bias+gelu, 3 bias+residual (fp32 accumulate, bf16 out)."""
    y = x.float() @ w.float().T
    if epi >= 1:
        y = y + bias.float()
    if epi == 2:
        y = F.gelu(y)
    if epi == 3:
        y = y + residual.float()
    return y.to(x.dtype)


def embedding(ids, table):
    return table[ids.long()]


def bert_embed_ln(ids, pos, token_type, wte, wpe, wtt, gamma, beta, eps):
    tt = token_type.long() if token_type is not None else torch.zeros_like(ids, dtype=torch.long)
    e = wte[ids.long()].float() + wpe[pos.long()].float() + wtt[tt].float()
    return F.layer_norm(e, (wte.shape[1],), gamma.float(), beta.float(), eps).to(wte.dtype)


def argmax(logits):
    return logits.float().argmax(dim=-1)


def token_cls_argmax(h, w, bias, n_valid):
    logits = h.float() @ w[:n_valid].float().t() + bias[:n_valid].float()
    return logits.argmax(dim=-1)


def sample(logits, inv_temp, top_k, top_p, u):
    out = torch.empty(logits.shape[0], dtype=torch.long, device=logits.device)
    for r in range(logits.shape[0]):
        x = logits[r].float() * float(inv_temp[r])
        k = int(top_k[r])
        if 0 < k < x.numel():
            th = torch.topk(x, k).values[-1]
            x = torch.where(x >= th, x, torch.full_like(x, -math.inf))
        p = torch.softmax(x, -1)
        tp = float(top_p[r])
        if 0.0 < tp < 1.0:
            sp, si = torch.sort(p, descending=True)
            keep = torch.cumsum(sp, 0) - sp < tp
            mask = torch.zeros_like(p, dtype=torch.bool)
            mask[si[keep]] = True
            p = torch.where(mask, p, torch.zeros_like(p))
            p = p / p.sum()
        c = torch.cumsum(p, 0)
        idx = int(torch.searchsorted(c, torch.tensor([float(u[r])], device=c.device)).clamp(max=x.numel() - 1))
        out[r] = idx
    return out


def paged_decode(q, k_cache, v_cache, block_tables, context_lens, Hq, max_context, scale):
    B = q.shape[0]
    NB, Hkv, BS, D = k_cache.shape
    G = Hq // Hkv
    out = torch.empty(B, Hq * D, dtype=q.dtype, device=q.device)
    for b in range(B):
        L = int(context_lens[b])
        nblk = (L + BS - 1) // BS
        blocks = block_tables[b, :nblk].long()
        k = k_cache[blocks].permute(1, 0, 2, 3).reshape(Hkv, nblk * BS, D)[:, :L].float()
        v = v_cache[blocks].permute(1, 0, 2, 3).reshape(Hkv, nblk * BS, D)[:, :L].float()
        qb = q[b, : Hq * D].view(Hkv, G, D).float()
        s = torch.einsum("hgd,htd->hgt", qb, k) * scale
        p = torch.softmax(s, -1)
        o = torch.einsum("hgt,htd->hgd", p, v)
        out[b] = o.reshape(-1).to(q.dtype)
    return out


def paged_decode_cascade(q, k_cache, v_cache, block_tables, context_lens, Hq, max_context, scale,
                         prefix_table, prefix_len, nchunk=8):
    """Cascade decode attention: keys [0, P) come from the shared ``prefix_table`` blocks,
    keys [P, L) from each sequence's own block table (one softmax over both)."""
    B = q.shape[0]
    NB, Hkv, BS, D = k_cache.shape
    G = Hq // Hkv
    P = int(prefix_len.reshape(-1)[0])
    pb = prefix_table.reshape(-1)[: P // BS].long()
    kp = k_cache[pb].permute(1, 0, 2, 3).reshape(Hkv, -1, D).float()
    vp = v_cache[pb].permute(1, 0, 2, 3).reshape(Hkv, -1, D).float()
    out = torch.zeros(B, Hq * D, dtype=q.dtype, device=q.device)
    for b in range(B):
        L = int(context_lens[b])
        if L <= P:
            continue
        nblk = (L + BS - 1) // BS
        blocks = block_tables[b, P // BS:nblk].long()
        ks = k_cache[blocks].permute(1, 0, 2, 3).reshape(Hkv, -1, D)[:, : L - P].float()
        vs = v_cache[blocks].permute(1, 0, 2, 3).reshape(Hkv, -1, D)[:, : L - P].float()
        k, v = torch.cat([kp, ks], 1), torch.cat([vp, vs], 1)
        qb = q[b, : Hq * D].view(Hkv, G, D).float()
        p = torch.softmax(torch.einsum("hgd,htd->hgt", qb, k) * scale, -1)
        out[b] = torch.einsum("hgt,htd->hgd", p, v).reshape(-1).to(q.dtype)
    return out


def flash_prefill(qkv, cu_seqlens, max_len, Hq, Hkv, D, scale, causal):
    T = qkv.shape[0]
    x = qkv.view(T, Hq + 2 * Hkv, D)
    G = Hq // Hkv
    out = torch.empty(T, Hq * D, dtype=qkv.dtype, device=qkv.device)
    cu = cu_seqlens.tolist()
    for b in range(len(cu) - 1):
        s0, s1 = cu[b], cu[b + 1]
        L = s1 - s0
        if L == 0:
            continue
        q = x[s0:s1, :Hq].float().transpose(0, 1)  # [Hq, L, D]
        k = x[s0:s1, Hq : Hq + Hkv].float().transpose(0, 1).repeat_interleave(G, 0)
        v = x[s0:s1, Hq + Hkv :].float().transpose(0, 1).repeat_interleave(G, 0)
        s = torch.einsum("hld,hmd->hlm", q, k) * scale
        if causal:
            mask = torch.ones(L, L, dtype=torch.bool, device=qkv.device).triu(1)
            s = s.masked_fill(mask, -math.inf)
        o = torch.einsum("hlm,hmd->hld", torch.softmax(s, -1), v)
        out[s0:s1] = o.transpose(0, 1).reshape(L, Hq * D).to(qkv.dtype)
    return out


def flash_prefill_paged(qkv, cu_seqlens, max_len, Hq, Hkv, D, scale, k_cache, v_cache,
                        block_tables, ctx_start):
    """Causal attention of the new tokens over (cached prefix + new) keys read from the
    paged cache (the new keys must already be written there)."""
    T = qkv.shape[0]
    x = qkv.view(T, Hq + 2 * Hkv, D)
    G = Hq // Hkv
    BS = k_cache.shape[2]
    out = torch.empty(T, Hq * D, dtype=qkv.dtype, device=qkv.device)
    cu = cu_seqlens.tolist()
    for b in range(len(cu) - 1):
        s0, s1 = cu[b], cu[b + 1]
        L = s1 - s0
        if L == 0:
            continue
        P0 = int(ctx_start[b])
        Lk = P0 + L
        nblk = (Lk + BS - 1) // BS
        blocks = block_tables[b, :nblk].long()
        k = k_cache[blocks].permute(1, 0, 2, 3).reshape(Hkv, nblk * BS, D)[:, :Lk].float()
        v = v_cache[blocks].permute(1, 0, 2, 3).reshape(Hkv, nblk * BS, D)[:, :Lk].float()
        k = k.repeat_interleave(G, 0)
        v = v.repeat_interleave(G, 0)
        q = x[s0:s1, :Hq].float().transpose(0, 1)
        s = torch.einsum("hld,hmd->hlm", q, k) * scale
        qpos = torch.arange(P0, Lk, device=qkv.device)[:, None]
        kpos = torch.arange(Lk, device=qkv.device)[None, :]
        s = s.masked_fill(kpos > qpos, -math.inf)
        o = torch.einsum("hlm,hmd->hld", torch.softmax(s, -1), v)
        out[s0:s1] = o.transpose(0, 1).reshape(L, Hq * D).to(qkv.dtype)
    return out


def knn(xb, xb_norms, xq, k, inner_product, id_offset):
    """FAISS IndexFlat semantics: L2 -> ascending squared distances, IP -> descending."""
    nq = xq.shape[0]
    N = xb.shape[0]
    D = torch.full((nq, k), -3.4028234663852886e38 if inner_product else 3.4028234663852886e38,
                   dtype=torch.float32, device=xq.device)
    I = torch.full((nq, k), -1, dtype=torch.long, device=xq.device)
    if N == 0 or nq == 0:
        return D, I
    xbf = xb.float()
    xqf = xq.float()
    ip = xqf @ xbf.T
    if inner_product:
        vals, idx = torch.topk(ip, min(k, N), dim=1, largest=True)
    else:
        norms = xb_norms.float() if xb_norms is not None else (xbf * xbf).sum(1)
        d = (xqf * xqf).sum(1, keepdim=True) + norms[None, :] - 2 * ip
        vals, idx = torch.topk(d, min(k, N), dim=1, largest=False)
    D[:, : vals.shape[1]] = vals
    I[:, : idx.shape[1]] = idx + id_offset
    return D, I


def pool_l2(h, cu_seqlens, mean, normalize):
    cu = cu_seqlens.tolist()
    out = torch.zeros(len(cu) - 1, h.shape[-1], dtype=torch.float32, device=h.device)
    for b in range(len(cu) - 1):
        s0, s1 = cu[b], cu[b + 1]
        if s1 > s0:
            out[b] = h[s0:s1].float().mean(0) if mean else h[s0].float()
    if normalize:
        out = F.normalize(out, dim=-1, eps=1e-12)
    return out


def decode_slots(block_tables, positions, valid, BS: int):
    blk = torch.gather(block_tables, 1, (positions // BS).long().clamp(max=block_tables.shape[1] - 1)[:, None])[:, 0]
    return torch.where(valid.bool(), blk * BS + positions % BS, torch.full_like(blk, -1)).int()


def decode_advance(nxt, out, tokens, positions, context_lens, valid) -> None:
    out.copy_(nxt)
    tokens.copy_(nxt.int())
    positions.add_(valid)
    context_lens.add_(valid)


def coarse_probes(xq, centroids, cnorm, nprobe: int):
    """fp32 reference of csrc/kernels/coarse.hip: ||c||^2 - 2 q.c per (query, centroid),
    the nprobe smallest in ascending order, ties to the lower centroid id (stable sort)."""
    d = cnorm.float()[None, :] - 2.0 * (xq.float() @ centroids.float().t())
    order = torch.sort(d, dim=1, stable=True).indices
    return order[:, :nprobe].contiguous()


# --------------------------------------------------- hybrid decoders (fp32 residual stream)
def _slab_sum(P):
    """The fp32 product of split-K slabs [S, M, N], or of the product [M, N] itself."""
    return P.float().sum(0) if P.dim() == 3 else P.float()


def _rms(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def sandwich_rmsnorm(P, residual, w_post, w_next, eps, add=None, out_dtype=None):
    residual.add_(_rms(_slab_sum(P), eps) * w_post)
    if add is not None:
        residual.add_(add)
    return (_rms(residual, eps) * w_next).to(out_dtype or residual.dtype)


def embed_scale_rmsnorm(ids, table, scale, w, eps, keep):
    h = table[ids.long()].float() * scale
    return h, (h.clone() if keep else None), (h if w is None else _rms(h, eps) * w).to(table.dtype, copy=True)


def scaled_rmsnorm(P, residual, scale, w_next, eps, bias, mix, out_dtype):
    if mix is None:
        y = _slab_sum(P)
    else:
        ids, wts, experts, x = mix
        y = sum(wts[:, k, None] * torch.where(ids[:, k, None] < experts, P[k].float(), x.float()) for k in range(P.shape[0]))
    residual.add_(scale * (y if bias is None else y + bias))
    return (_rms(residual, eps) * w_next).to(out_dtype or residual.dtype)


def poly_norm(P, bias, act, n_out, eps, out_dtype):
    z = _slab_sum(P)[:, :bias.shape[0]] + bias
    y = sum(act[i] * _rms(z.pow(i + 1), eps) for i in range(3)) + act[3]
    return F.pad(y, (0, n_out - y.shape[1])).to(out_dtype)


def activation(P, act, out_dtype):
    x = _slab_sum(P)
    return (F.gelu(x, approximate="tanh") if act == "gelu_tanh" else x.clamp(min=0).square()).to(out_dtype)


def add_scaled(P, Q, residual, m, out_dtype):
    y = _slab_sum(P)
    residual.add_((y if Q is None else y + _slab_sum(Q)) * m)
    return residual.to(out_dtype)


def side_gate(P, ids, table, col, n, out_dtype):
    x = _slab_sum(P)
    e = torch.zeros_like(x)
    e[:, :n] = table[ids.long(), col:col + n].float()
    return (F.gelu(x, approximate="tanh") * e).to(out_dtype)


def soft_cap(x, cap):
    return cap * torch.tanh(x.float() / cap)


def rope_table(positions, inv_freq, mult=1.0):
    a = positions.double()[:, None] * inv_freq
    return (torch.cat([a.cos(), a.sin()], -1) * mult).float()


def _rotate(x, cs):
    """x [T, ..., r] by the [cos | sin] rows cs [T, r], dimension i paired with i + r / 2."""
    h = x.shape[-1] // 2
    cs = cs.view(cs.shape[0], *[1] * (x.dim() - 2), 2 * h)
    u, v, c, s = x[..., :h], x[..., h:], cs[..., :h], cs[..., h:]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def latent_store(P, cs, slots, cache, c_norm, H, dim, rank, eps, dtype):
    x = _slab_sum(P)
    T, r = cs.shape
    d8, r8 = -(-dim // 8) * 8, -(-r // 8) * 8
    q = torch.zeros(T, H, d8 + r8, dtype=dtype, device=x.device)
    xq = x[:, :H * (dim + r)].view(T, H, dim + r)
    q[..., :dim] = xq[..., :dim].to(dtype)
    q[..., d8:d8 + r] = _rotate(xq[..., dim:], cs).to(dtype)
    if c_norm is not None:
        _store_latent(x[:, H * (dim + r):], cs, slots, cache, c_norm, eps)
    return q.view(T, H * (d8 + r8))


def _store_latent(x, cs, slots, cache, c_norm, eps):
    """The cache row of [latent | key part | ..]."""
    (T, r), rank = cs.shape, c_norm.shape[0]
    BS, D = cache.shape[2:]
    r8 = -(-r // 8) * 8
    row = torch.zeros(T, D, dtype=cache.dtype, device=x.device)
    row[:, :rank] = (_rms(x[:, :rank], eps) * c_norm).to(cache.dtype)
    row[:, D - r8:D - r8 + r] = _rotate(x[:, rank:rank + r], cs).to(cache.dtype)
    sm = slots.long()
    ok = sm >= 0
    cache[sm[ok] // BS, 0, sm[ok] % BS] = row[ok]


def latent_norm_store(P, cs, slots, cache, q_norm, c_norm, eps, dtype):
    x, n = _slab_sum(P), q_norm.shape[0]
    _store_latent(x[:, n:], cs, slots, cache, c_norm, eps)
    return (_rms(x[:, :n], eps) * q_norm).to(dtype)


def head_gate(x, P, col, per, row):
    T, n = x.shape
    g = torch.sigmoid(_slab_sum(P)[row:row + T, col:col + n // per])
    return (x.float().view(T, -1, per) * g[..., None]).view(T, n).to(x.dtype)


def head_project(x, w, carry):
    H, N, K = w.shape
    T = x.shape[0]
    xh = x.view(T, H, -1)
    y = torch.matmul(xh[..., :K].float().transpose(0, 1), w.float().transpose(1, 2)).transpose(0, 1).to(x.dtype)
    return torch.cat([y, xh[..., K:K + carry]], -1).reshape(T, H * (N + carry)) if carry else y.reshape(T, H * N)


def qk_norm_store(P, w, slots, k_cache, k_scale, H, eps):
    x = _slab_sum(P)
    T = x.shape[0]
    NB, G, BS, D = k_cache.shape
    q = (_rms(x[:, :H * D].view(T, H, D), eps) * w).to(k_cache.dtype).reshape(T, H * D)
    k = x[:, H * D:(H + G) * D].reshape(T, G, D).to(k_cache.dtype)
    sm = slots.long()
    ok = sm >= 0
    blk, off = sm[ok] // BS, sm[ok] % BS
    k_cache[blk, :, off] = k[ok]
    k_scale.view(NB, G, BS)[blk, :, off] = torch.rsqrt(k[ok].float().pow(2).mean(-1) + eps)
    return q


def window_attn(q, k_cache, v_cache, k_scale, block_tables, cu, ctx, scale, window, sink, v_dim, cap=0.0, out_scale=1.0,
                out=None):
    NB, G, BS, D = k_cache.shape
    H = q.shape[1] // D
    v_cache = k_cache if v_cache is None else v_cache
    v_dim = v_dim or v_cache.shape[3]
    out = q.new_zeros(q.shape[0], H * v_dim) if out is None else out
    for b in range(block_tables.shape[0]):
        q0, L, p0 = (b, 1, int(ctx[b]) - 1) if cu is None else (int(cu[b]), int(cu[b + 1] - cu[b]), int(ctx[b]))
        if L <= 0 or p0 < 0:
            continue
        n = p0 + L
        lo = max(0, p0 - window + 1) if window > 0 else 0
        pos = torch.arange(lo, n, device=q.device)
        blk, off = block_tables[b, (pos // BS)].long(), pos % BS
        k = k_cache[blk, :, off].float().transpose(0, 1)                # [G, keys, D]
        v = v_cache[blk, :, off, :v_dim].float().transpose(0, 1)
        qb = q[q0:q0 + L].view(L, G, H // G, D).float().permute(1, 2, 0, 3)
        s = torch.einsum("ghld,gkd->ghlk", qb, k) * scale
        if k_scale is not None:
            s = s * k_scale.view(NB, G, BS)[blk, :, off].t()[:, None, None, :]
        if cap:
            s = cap * torch.tanh(s / cap)
        i = torch.arange(p0, n, device=q.device)[:, None]
        dead = pos[None, :] > i
        if window > 0:
            dead = dead | (pos[None, :] <= i - window)
        s = s.masked_fill(dead, -math.inf)
        if sink is not None:
            s = torch.cat([s, sink.float().view(G, H // G, 1, 1).expand(G, H // G, L, 1)], -1)
        p = torch.softmax(s, -1)[..., :n - lo]
        o = torch.einsum("ghlk,gkd->ghld", p, v)
        out[q0:q0 + L] = (o.permute(2, 0, 1, 3).reshape(L, H * v_dim) * out_scale).to(q.dtype)
    return out


def latent_gather(cache, block_tables, first, cu_k, total, rank):
    BS, D = cache.shape[2:]
    out = cache.new_zeros(total, D)
    for b in range(block_tables.shape[0]):
        k0, n = int(first[b]), int(cu_k[b + 1] - cu_k[b])
        pos = torch.arange(k0, k0 + n, device=cache.device)
        out[int(cu_k[b]):int(cu_k[b + 1])] = cache[block_tables[b, pos // BS].long(), 0, pos % BS]
    return out[:, :rank].contiguous(), out[:, rank:].contiguous()


def packed_window_attn(q, kv, kr, H, dim, vdim, cu, cu_k, scale, window, sink):
    r8 = kr.shape[1]
    d8, v8 = -(-dim // 8) * 8, -(-vdim // 8) * 8
    out = q.new_zeros(q.shape[0], H * vdim)
    for b in range(cu.numel() - 1):
        q0, L, k0, n = int(cu[b]), int(cu[b + 1] - cu[b]), int(cu_k[b]), int(cu_k[b + 1] - cu_k[b])
        if L <= 0:
            continue
        qb = q[q0:q0 + L].view(L, H, d8 + r8).float()
        k = kv[k0:k0 + n, :H * d8].view(n, H, d8).float()
        v = kv[k0:k0 + n, H * d8:H * (d8 + v8)].view(n, H, v8).float()
        s = torch.einsum("lhd,khd->hlk", qb[..., :d8], k) + torch.einsum("lhr,kr->hlk", qb[..., d8:], kr[k0:k0 + n].float())
        i, j = torch.arange(n - L, n, device=q.device)[:, None], torch.arange(n, device=q.device)[None]
        dead = (j > i) | (j <= i - window) if window > 0 else j > i
        s = (s * scale).masked_fill(dead, -math.inf)
        if sink is not None:
            s = torch.cat([s, sink.float().view(H, 1, 1).expand(H, L, 1)], -1)
        p = torch.softmax(s, -1)[..., :n]
        out[q0:q0 + L] = torch.einsum("hlk,khd->lhd", p, v)[..., :vdim].reshape(L, H * vdim).to(q.dtype)
    return out


def causal_conv(x, w, bias, state, slots, cu, ctx, silu=True):
    taps, C = w.shape
    y = torch.empty(x.shape[0], C, dtype=x.dtype, device=x.device)
    for b in range(cu.numel() - 1):
        q0, q1, slot = int(cu[b]), int(cu[b + 1]), int(slots[b])
        if q1 <= q0:
            continue
        head = (state[slot] if slot >= 0 and int(ctx[b]) > 0
                else torch.zeros(taps - 1, C, dtype=x.dtype, device=x.device))
        seq = torch.cat([head, x[q0:q1, :C]])
        acc = (w.new_zeros(C) if bias is None else bias).expand(q1 - q0, C).clone()
        for k in range(taps):
            acc += w[k] * seq[k:k + q1 - q0].float()
        y[q0:q1] = (F.silu(acc) if silu else acc).to(x.dtype)
        if slot >= 0 and taps > 1:
            state[slot] = seq[-(taps - 1):]
    return y


def conv_step(P, w, bias, state, slots, positions, silu=True, rest=-1):
    C = w.shape[1]
    B = P.shape[-2]
    xz = _slab_sum(P).to(state.dtype)
    xz = xz if rest < 0 else xz[:, :C + rest]
    cu = torch.arange(B + 1, dtype=torch.int32)
    y = causal_conv(xz[:, :C], w, bias, state, slots, cu, positions, silu)
    return y, (xz[:, C:].contiguous() if xz.shape[1] > C else None)


def selective_scan(x, dt, bc, b_off, c_off, N, z, A2, D, dt_b, state, slots, cu, ctx):
    C, Np = A2.shape
    y = torch.empty_like(x)
    d = F.softplus(dt.float() + dt_b)
    xf = x.float()
    Bv, Cv = F.pad(bc[:, b_off:b_off + N].float(), (0, Np - N)), F.pad(bc[:, c_off:c_off + N].float(), (0, Np - N))
    for b in range(cu.numel() - 1):
        q0, q1, slot = int(cu[b]), int(cu[b + 1]), int(slots[b])
        S = (state[slot].clone() if slot >= 0 and int(ctx[b]) > 0 else torch.zeros(C, Np, device=x.device))
        for t in range(q0, q1):
            S = torch.exp2(d[t][:, None] * A2) * S + (d[t] * xf[t])[:, None] * Bv[t]
            y[t] = ((S @ Cv[t] + D * xf[t]) * F.silu(z[t, :C].float())).to(x.dtype)
        if slot >= 0 and q1 > q0:
            state[slot] = S
    return y


def selective_step(x, dt, bc, b_off, c_off, N, z, A2, D, dt_b, state, slots, positions):
    cu = torch.arange(x.shape[0] + 1, dtype=torch.int32)
    return selective_scan(x, dt, bc, b_off, c_off, N, z, A2, D, dt_b, state, slots, cu, positions)


# ------------------------------------------- attention with rotated keys, linear attention
def qkv_rope_store(P, bias, qw, kw, cs, slots, k_cache, v_cache, H, eps):
    x = _slab_sum(P)
    T = x.shape[0]
    G, BS, D = k_cache.shape[1:]
    DV = v_cache.shape[3]
    n = (H + G) * D + G * DV
    x = x[:, :n] + bias if bias is not None else x[:, :n]
    q, k = x[:, :H * D].reshape(T, H, D), x[:, H * D:(H + G) * D].reshape(T, G, D)
    r = cs.shape[1]

    def head(y, w):
        y = _rms(y, eps) * w if w is not None else y
        return torch.cat([_rotate(y[..., :r], cs), y[..., r:]], -1).to(k_cache.dtype) if r else y.to(k_cache.dtype)

    sm = slots.long()
    ok = sm >= 0
    blk, off = sm[ok] // BS, sm[ok] % BS
    k_cache[blk, :, off] = head(k, kw)[ok]
    v_cache[blk, :, off] = x[:, (H + G) * D:].reshape(T, G, DV).to(v_cache.dtype)[ok]
    return head(q, qw).reshape(T, H * D)


def _linear_inputs(X, Z, m, w_gate, b_gate, cs):
    """fp32 (q, k [T, H, d], v, gate [T, H, vd], log decay [T, H, d or 1], beta [T, H] or None)."""
    x, z = _slab_sum(X), _slab_sum(Z)
    T, H, G, d, vd = x.shape[0], m.heads, m.kv_heads, m.dim, m.vdim

    def cols(t, at, h, n):
        return t[:, at:at + h * n].reshape(T, h, n)

    q, k, v, g = cols(x, m.q, G, d), cols(x, m.k, G, d), cols(x, m.v, H, vd), cols(z, m.g, H, vd)
    beta = None
    if m.kind == "delta":
        q, k = (t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) + 1e-6) for t in (q, k))
        la = (w_gate * F.softplus(z[:, m.a:m.a + H] + b_gate))[..., None]
        beta = torch.sigmoid(z[:, m.b:m.b + H])
    elif m.kind == "channel_delta":
        q, k = (t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) + 1e-6) for t in (q, k))
        la = w_gate[:, None] * F.softplus(z[:, m.a:m.a + H * d] + b_gate).view(T, H, d)
        beta = torch.sigmoid(z[:, m.b:m.b + H])
    elif m.kind == "channel":
        la = (F.logsigmoid(z[:, m.a:m.a + m.rank] @ w_gate.t() + b_gate) * m.inv_tau).view(T, H, d)
    else:
        r = cs.shape[1]
        q, k = (torch.cat([_rotate(t[..., :r], cs), t[..., r:]], -1) for t in (q, k))
        la = w_gate.view(1, H, 1).expand(T, H, 1)
    q, k = (t.repeat_interleave(H // G, 1) for t in (q * m.q_scale, k * m.k_scale))
    return q, k, v, g, la, beta


def linear_scan(X, Z, m, w_gate, b_gate, cs, norm, state, slots, cu, ctx, out):
    q, k, v, g, la, beta = _linear_inputs(X, Z, m, w_gate, b_gate, cs)
    H, d, vd = m.heads, m.dim, m.vdim
    gate = torch.sigmoid if m.gate == "sigmoid" else F.silu
    for b in range(cu.numel() - 1):
        q0, q1, slot = int(cu[b]), int(cu[b + 1]), int(slots[b])
        if q1 <= q0:
            continue
        S = (state[slot, ..., :vd].clone() if slot >= 0 and int(ctx[b]) > 0
             else torch.zeros(H, d, vd, device=state.device))
        for t in range(q0, q1):
            S = torch.exp(la[t])[..., None] * S
            u = v[t] if beta is None else beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
            S = S + k[t][..., None] * u[:, None]
            o = torch.einsum("hdv,hd->hv", S, q[t])
            out[t] = (_rms(o, m.eps) * norm * gate(g[t])).reshape(-1).to(out.dtype)
        if slot >= 0:
            state[slot, ..., :vd] = S
    return out


def linear_step(X, Z, m, w_gate, b_gate, cs, norm, state, slots, positions, out):
    n = X.shape[-2]
    return linear_scan(X, Z, m, w_gate, b_gate, cs, norm, state, slots, torch.arange(n + 1, dtype=torch.int32), positions, out)


def low_rank(Z, at, w_a, w_g, n):
    ka, kg = w_a.shape[1], w_g.shape[1]
    z = Z[:, at:at + ka + kg + n]
    return torch.cat([z[:, :ka].float() @ w_a.float().t(), z[:, ka:ka + kg].float() @ w_g.float().t(), z[:, ka + kg:].float()], -1)


# ------------------------------------------------------------ norms after the sum, experts
def post_norm(P, Q, gate, col, gate_b, res, alpha, w, groups, eps, out_dtype):
    x = alpha * res
    if P is not None:
        y = _slab_sum(P)
        if Q is not None:
            y = y + _slab_sum(Q)
        x = x + torch.sigmoid(_slab_sum(gate)[:, col:col + res.shape[1]] + gate_b) * y
    T, W = res.shape
    res.copy_(_rms(x.view(T, groups, W // groups), eps).view(T, W) * w)
    return res.to(out_dtype)


def moe_route(x, w, experts, top):
    z = x.float() @ w.float().t()
    s = torch.sigmoid(z)
    best = torch.topk(s[:, :experts], top, -1)
    return best.indices.to(torch.int32), best.values, s[:, experts:].contiguous()


def moe_route_groups(x, w, correction, top, groups, keep, scale):
    s = torch.softmax(x.float() @ w.float().t(), -1)
    choice = s + correction
    T, N = s.shape
    parts = choice.view(T, groups, N // groups)
    best = torch.topk(parts.amax(-1), keep, -1).indices
    alive = torch.zeros(T, groups, dtype=torch.bool, device=x.device).scatter_(1, best, True)
    ids = torch.topk(parts.masked_fill(~alive[..., None], -math.inf).reshape(T, N), top, -1).indices
    wts = s.gather(1, ids)
    return ids.to(torch.int32), wts / (wts.sum(-1, keepdim=True) + 1e-20) * scale


def glu(P, col, n, scale, out_dtype):
    x = _slab_sum(P)
    y = F.silu(x[:, col:col + n]) * x[:, col + n:col + 2 * n]
    return (y if scale is None else y * scale.view(-1, 1)).to(out_dtype)


def moe_experts(x, ids, wts, up, down, limit=0.0):
    T, top = ids.shape
    out = torch.zeros(top, T, down.shape[1], dtype=x.dtype, device=x.device)
    for e in range(up.shape[0]):
        t, k = (ids == e).nonzero(as_tuple=True)
        if t.numel() == 0:
            continue
        g, u = x[t].float() @ up[e, 0].float().t(), x[t].float() @ up[e, 1].float().t()
        if limit > 0:
            g, u = g.clamp(max=limit), u.clamp(-limit, limit)
            a = (g * torch.sigmoid(1.702 * g) * (u + 1)).to(x.dtype)
        else:
            s = wts[t, k][:, None]
            a = (F.silu(s * g) * (s * u)).to(x.dtype)
        out[k, t] = (a.float() @ down[e].float().t()).to(x.dtype)
    return out
