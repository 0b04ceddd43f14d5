"""Plain-PyTorch reference implementations of every engine op.

These are (1) the numerics oracle the HIP kernels are tested against
(fp32 math, same data layouts, same masking rules) and (2) the compute path
on CPU-only hosts, where the tiny test models run.  On a GPU the engine uses
``ops.hip`` exclusively (see ``ops/__init__.py``).

Layouts shared with the kernels (``csrc/kernels/*.hip``):

* ``qkv`` [T, (Hq + 2 Hkv) * D]: Q heads, then K heads, then V heads.
* KV cache per layer: ``kcache``/``vcache`` [num_pages, Hkv, P, D];
  token at position ``p`` of a sequence lives in page
  ``block_tables[row, p // P]`` at offset ``p % P``.
* ``cos_sin`` [max_pos, D/2, 2] fp32 (cos, sin), HF rotate-half pairing.
* fp8 KV cache (``--kv-dtype fp8``: K and V; ``fp8v``: V only, K stays bf16; csrc/kernels/kv8.h): per layer uint8 [num_pages, Hkv, SLAB],
  SLAB = P * D + 4 * P -- a (page, head) slab holds P rows of D e4m3fn bytes, then P fp32 row scales;
  a row is quantised whole with the power-of-two scale >= max|x| / 448.
"""

from __future__ import annotations

import math
from typing import Optional

import torch

LOG2E = 1.4426950408889634


def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    xf = x.float()
    y = xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    y = y.to(x.dtype)
    if out is not None:
        out.copy_(y)
        return out
    return y


def add_rmsnorm(x: torch.Tensor, residual: torch.Tensor, w: torch.Tensor, eps: float,
                out: Optional[torch.Tensor] = None) -> torch.Tensor:
    residual.copy_((x.float() + residual.float()).to(residual.dtype))
    return rmsnorm(residual, w, eps, out)


def rope_inv_freq(head_dim: int, theta: float, scaling=None) -> torch.Tensor:
    """RoPE inverse frequencies (float64); ``scaling`` = (factor, low_freq_factor, high_freq_factor,
    original_max_position) applies Llama-3.1's "llama3" rule: wavelengths longer than
    orig / low_freq_factor are divided by ``factor``, shorter than orig / high_freq_factor kept, and the
    band between interpolated smoothly."""
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    if scaling is None:
        return inv
    factor, low, high, orig = scaling
    wavelen = 2 * math.pi / inv
    low_wl, high_wl = orig / low, orig / high
    smooth = ((orig / wavelen) - low) / (high - low)
    mid = (1 - smooth) * inv / factor + smooth * inv
    out = torch.where(wavelen > low_wl, inv / factor, inv)
    band = (wavelen <= low_wl) & (wavelen >= high_wl)
    return torch.where(band, mid, out)


def rope_cos_sin(max_pos: int, head_dim: int, theta: float, device=None, scaling=None) -> torch.Tensor:
    inv = rope_inv_freq(head_dim, theta, scaling)
    t = torch.arange(max_pos, dtype=torch.float64)
    ang = torch.outer(t, inv)
    return torch.stack([ang.cos(), ang.sin()], dim=-1).float().contiguous().to(device)


def kv8_slab(page: int, d: int) -> int:
    return page * d + 4 * page


def kv8_quant_rows(x: torch.Tensor):
    """Rows [..., d] -> (e4m3fn bytes [..., d] uint8, fp32 scales [...]): scale = the power of two >= max|x| / 448
    (1 for a zero row) and at least 2^-126 (a normal number: 1 / scale stays finite), q = RNE e4m3(x / scale) --
    kv8.h's row rule."""
    xf = x.float()
    amax = xf.abs().amax(-1)
    m, e = torch.frexp(amax / 448.0)
    e = torch.clamp(torch.where(m == 0.5, e - 1, e), min=-126)
    sc = torch.where(amax > 0, torch.ldexp(torch.ones_like(amax), e), torch.ones_like(amax))
    q = (xf / sc[..., None]).to(torch.float8_e4m3fn).view(torch.uint8)
    return q, sc


def kv8_from_bf16(cache: torch.Tensor) -> torch.Tensor:
    """A bf16 cache [pages, Hkv, P, d] in the fp8 slab layout [pages, Hkv, P * d + 4 P] (every row quantised)."""
    n, hkv, page, d = cache.shape
    q, sc = kv8_quant_rows(cache)
    return torch.cat([q.reshape(n, hkv, page * d), sc.contiguous().view(torch.uint8).reshape(n, hkv, 4 * page)], -1)


def cache_pages(cache: torch.Tensor, pages: torch.Tensor, page: int, d: int) -> torch.Tensor:
    """fp32 [len(pages), Hkv, P, d] of a bf16 or fp8-slab cache."""
    c = cache.index_select(0, pages)
    if cache.dtype != torch.uint8:
        return c.float()
    q = c[..., : page * d].reshape(*c.shape[:2], page, d).contiguous().view(torch.float8_e4m3fn).float()
    sc = c[..., page * d:].contiguous().view(torch.float32)
    return q * sc[..., None]


def cache_write(cache: torch.Tensor, pages: torch.Tensor, offs: torch.Tensor, rows: torch.Tensor, page: int,
                d: int) -> None:
    """cache[pages[i], :, offs[i]] = rows[i] ([n, Hkv, d]) for a bf16 or fp8-slab cache."""
    if cache.dtype != torch.uint8:
        cache[pages, :, offs] = rows.to(cache.dtype)
        return
    q, sc = kv8_quant_rows(rows)  # [n, Hkv, d] bytes, [n, Hkv]
    n, hkv = rows.shape[0], rows.shape[1]
    col = offs[:, None] * d + torch.arange(d, device=offs.device)[None, :]  # [n, d] byte columns
    for h in range(hkv):
        cache[pages[:, None], h, col] = q[:, h]
        sb = page * d + 4 * offs[:, None] + torch.arange(4, device=offs.device)[None, :]
        cache[pages[:, None], h, sb] = sc[:, h].contiguous().view(torch.uint8).view(n, 4)


def rope_kv(qkv: torch.Tensor, positions: torch.Tensor, seq_idx: torch.Tensor, block_tables: torch.Tensor,
            kcache: Optional[torch.Tensor], vcache: Optional[torch.Tensor], cos_sin: torch.Tensor,
            hq: int, hkv: int, d: int, page: int, write_cache: bool = True) -> None:
    T = qkv.shape[0]
    if T == 0:
        return
    half = d // 2
    pos = positions[:T].long()
    cs = cos_sin[pos]  # [T, half, 2]
    cos, sin = cs[..., 0][:, None, :], cs[..., 1][:, None, :]
    qk = qkv[:, : (hq + hkv) * d].view(T, hq + hkv, d).float()
    a, b = qk[..., :half], qk[..., half:]
    ra = a * cos - b * sin
    rb = b * cos + a * sin
    rot = torch.cat([ra, rb], dim=-1).to(qkv.dtype)
    qkv[:, : (hq + hkv) * d] = rot.reshape(T, -1)
    if write_cache:
        rows = seq_idx[:T].long()
        keep = rows >= 0  # seq_idx < 0: prefill padding token, never cached
        rows, p_, k = rows[keep], pos[keep], rot[:, hq:][keep]
        pages = block_tables[rows, p_ // page].long()
        offs = p_ % page
        v = qkv[:, (hq + hkv) * d: (hq + 2 * hkv) * d].view(T, hkv, d)[keep]
        cache_write(kcache, pages, offs, k, page, d)
        cache_write(vcache, pages, offs, v, page, d)


def rope_kv_parts(parts: torch.Tensor, positions, seq_idx, block_tables, kcache, vcache, cos_sin, hq, hkv, d, page,
                  out: Optional[torch.Tensor] = None) -> torch.Tensor:
    qkv = parts.float().sum(0).to(torch.bfloat16)
    rope_kv(qkv, positions, seq_idx, block_tables, kcache, vcache, cos_sin, hq, hkv, d, page)
    if out is not None:
        out.copy_(qkv)
        return out
    return qkv


def kv_scatter(rows: torch.Tensor, page: torch.Tensor, slot: torch.Tensor, kcache: torch.Tensor,
               vcache: torch.Tensor) -> None:
    """Reference of ops.hip.kv_scatter: cache[page[i], :, slot[i], :] = rows[i, 0 | 1] (page < 0 skipped)."""
    if kcache.dtype == torch.uint8 or vcache.dtype == torch.uint8:
        raise ValueError("kv_scatter: the context-parallel K/V exchange takes bf16 caches only")
    keep = page[: rows.shape[0]].long() >= 0
    pg, sl, r = page[: rows.shape[0]].long()[keep], slot[: rows.shape[0]].long()[keep], rows[keep]
    kcache[pg, :, sl, :] = r[:, 0].to(kcache.dtype)
    vcache[pg, :, sl, :] = r[:, 1].to(vcache.dtype)


def interleave_gate_up(wg: torch.Tensor, wu: torch.Tensor) -> torch.Tensor:
    """[F, H] gate + [F, H] up -> [2F, H] rows in blocks of 16 = [8 gate | 8 up]."""
    f, h = wg.shape
    return torch.stack([wg.reshape(f // 8, 8, h), wu.reshape(f // 8, 8, h)], dim=1).reshape(2 * f, h)


def split_gate_up(gu: torch.Tensor):
    """Inverse of the blocked column layout of a gate_up GEMM output."""
    f = gu.shape[-1] // 2
    v = gu.reshape(*gu.shape[:-1], f // 8, 2, 8)
    return v[..., 0, :].reshape(*gu.shape[:-1], f), v[..., 1, :].reshape(*gu.shape[:-1], f)


def swiglu(gu: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    g, u = split_gate_up(gu)
    g, u = g.float(), u.float()
    y = (g * torch.sigmoid(g) * u).to(gu.dtype)
    if out is not None:
        out.copy_(y)
        return out
    return y


class Fp8Weight:
    """OCP e4m3fn weight [N, K] with one fp32 scale per output row (W = scale[:, None] * float(q))."""

    def __init__(self, q: torch.Tensor, scale: torch.Tensor):
        self.q, self.scale = q, scale

    @property
    def shape(self):
        return self.q.shape

    def numel(self) -> int:
        return self.q.numel()

    def nbytes(self) -> int:
        return self.q.numel() + 4 * self.scale.numel()

    def dequant(self, dtype=torch.float32) -> torch.Tensor:
        return (self.q.float() * self.scale.float()[:, None]).to(dtype)

    @staticmethod
    def quantize(w: torch.Tensor) -> "Fp8Weight":
        wf = w.float()
        scale = wf.abs().amax(dim=1).clamp_min(1e-12) / 448.0
        q = (wf / scale[:, None]).clamp(-448.0, 448.0).to(torch.float8_e4m3fn)
        return Fp8Weight(q.contiguous(), scale.contiguous())


def _w(w):
    return w.dequant(torch.bfloat16) if isinstance(w, Fp8Weight) else w


def linear(x: torch.Tensor, w) -> torch.Tensor:
    if isinstance(w, Fp8Weight):
        return (x.float() @ w.dequant().t()).to(x.dtype)
    return torch.nn.functional.linear(x, w)


def linear_parts(x: torch.Tensor, w: torch.Tensor, splits: int = 1) -> torch.Tensor:
    """fp32 split-K partial slabs [S, M, N] of x @ w^T (what skinny_gemm EPI_F32_PARTIAL emits)."""
    K = x.shape[1]
    ks = K // splits
    wf = w.dequant() if isinstance(w, Fp8Weight) else w.float()
    return torch.stack([x[:, i * ks:(i + 1) * ks].float() @ wf[:, i * ks:(i + 1) * ks].t()
                        for i in range(splits)])


def linear_swiglu(x: torch.Tensor, w_gu) -> torch.Tensor:
    return swiglu(linear(x, w_gu))


def add_rmsnorm_parts(parts: torch.Tensor, residual: torch.Tensor, w: torch.Tensor, eps: float,
                      out: Optional[torch.Tensor] = None) -> torch.Tensor:
    residual.copy_((parts.float().sum(0) + residual.float()).to(residual.dtype))
    return rmsnorm(residual, w, eps, out)


def embed(ids: torch.Tensor, table: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    y = table[ids.long().clamp(0, table.shape[0] - 1)]
    if out is not None:
        out.copy_(y)
        return out
    return y


def attn_prefill(qkv: torch.Tensor, cu_seqlens: torch.Tensor, hq: int, hkv: int, d: int, scale: float,
                 out: Optional[torch.Tensor] = None) -> torch.Tensor:
    T = qkv.shape[0]
    if out is None:
        out = torch.empty(T, hq * d, dtype=qkv.dtype, device=qkv.device)
    cu = cu_seqlens.tolist()
    g = hq // hkv
    for i in range(len(cu) - 1):
        s, e = cu[i], cu[i + 1]
        if e <= s:
            continue
        n = e - s
        q = qkv[s:e, : hq * d].view(n, hq, d).float().transpose(0, 1)
        k = qkv[s:e, hq * d: (hq + hkv) * d].view(n, hkv, d).float().transpose(0, 1)
        v = qkv[s:e, (hq + hkv) * d: (hq + 2 * hkv) * d].view(n, hkv, d).float().transpose(0, 1)
        k = k.repeat_interleave(g, dim=0)
        v = v.repeat_interleave(g, dim=0)
        sc = torch.matmul(q, k.transpose(1, 2)) * scale
        mask = torch.ones(n, n, dtype=torch.bool, device=qkv.device).triu(1)
        sc.masked_fill_(mask, float("-inf"))
        p = torch.softmax(sc, dim=-1)
        o = torch.matmul(p, v).transpose(0, 1).reshape(n, hq * d)
        out[s:e] = o.to(out.dtype)
    return out


def attn_prefill_paged(qkv: torch.Tensor, cu_seqlens: torch.Tensor, hq: int, hkv: int, d: int, scale: float,
                       paged, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Chunked prefill: slice rows of every packed sequence attend to the cached positions
    [0, prefix) of that sequence (paged cache, already holding this slice's K/V too) and causally
    within the slice."""
    T = qkv.shape[0]
    if out is None:
        out = torch.empty(T, hq * d, dtype=qkv.dtype, device=qkv.device)
    cu = cu_seqlens.tolist()
    g = hq // hkv
    P = 64 if paged.kcache.dtype == torch.uint8 else paged.kcache.shape[2]
    for i in range(len(cu) - 1):
        s, e = cu[i], cu[i + 1]
        if e <= s:
            continue
        n, pre, slot = e - s, paged.prefix_host[i], paged.slot_host[i]
        tot = pre + n
        pages = paged.block_tables[slot, : -(-tot // P)].long()
        k = cache_pages(paged.kcache, pages, P, d).permute(1, 0, 2, 3).reshape(hkv, -1, d)[:, :tot]
        v = cache_pages(paged.vcache, pages, P, d).permute(1, 0, 2, 3).reshape(hkv, -1, d)[:, :tot]
        q = qkv[s:e, : hq * d].view(n, hq, d).float().transpose(0, 1)
        k = k.repeat_interleave(g, dim=0)
        v = v.repeat_interleave(g, dim=0)
        sc = torch.matmul(q, k.transpose(1, 2)) * scale
        qpos = torch.arange(pre, tot, device=qkv.device)[:, None]
        kpos = torch.arange(tot, device=qkv.device)[None, :]
        sc.masked_fill_(kpos > qpos, float("-inf"))
        p = torch.softmax(sc, dim=-1)
        out[s:e] = torch.matmul(p, v).transpose(0, 1).reshape(n, hq * d).to(out.dtype)
    return out


def attn_decode(q: torch.Tensor, kcache: torch.Tensor, vcache: torch.Tensor, block_tables: torch.Tensor,
                positions: torch.Tensor, hq: int, hkv: int, d: int, page: int, scale: float,
                out: Optional[torch.Tensor] = None, num_splits: int = 1) -> torch.Tensor:
    """q: [B, >= hq*d] (rows of the qkv buffer); context = positions + 1."""
    B = q.shape[0]
    if out is None:
        out = torch.empty(B, hq * d, dtype=q.dtype, device=q.device)
    g = hq // hkv
    for b in range(B):
        ctx = int(positions[b]) + 1
        npg = (ctx + page - 1) // page
        pages = block_tables[b, :npg].long()
        k = cache_pages(kcache, pages, page, d).permute(1, 0, 2, 3).reshape(hkv, npg * page, d)[:, :ctx]
        v = cache_pages(vcache, pages, page, d).permute(1, 0, 2, 3).reshape(hkv, npg * page, d)[:, :ctx]
        qq = q[b, : hq * d].view(hkv, g, d).float()
        sc = torch.matmul(qq, k.transpose(1, 2)) * scale
        p = torch.softmax(sc, dim=-1)
        o = torch.matmul(p, v).reshape(hq * d)
        out[b] = o.to(out.dtype)
    return out


# ----------------------------------------------------------------- sampler
_M1 = 0xbf58476d1ce4e5b9
_M2 = 0x94d049bb133111eb
_GOLD = 0x9E3779B97F4A7C15
_TOKMUL = 0xD1B54A32D192ED03
_U64 = (1 << 64) - 1


def _s64(x: int) -> int:
    x &= _U64
    return x - (1 << 64) if x >= (1 << 63) else x


def _lsr(x: torch.Tensor, n: int) -> torch.Tensor:
    return (x >> n) & ((1 << (64 - n)) - 1)


def _mix64_t(x: torch.Tensor) -> torch.Tensor:
    x = x ^ _lsr(x, 30)
    x = x * _s64(_M1)
    x = x ^ _lsr(x, 27)
    x = x * _s64(_M2)
    x = x ^ _lsr(x, 31)
    return x


def gumbel_noise(seed: int, position: int, vocab: int, device=None) -> torch.Tensor:
    """The sampler kernel's counter-based Gumbel noise for one row (fp32)."""
    k0 = _mix64_t(torch.tensor([_s64(seed * _GOLD + position + 1)], dtype=torch.int64))
    tok = torch.arange(vocab, dtype=torch.int64)
    h = _mix64_t(k0 ^ (tok * _s64(_TOKMUL)))
    u = (_lsr(h, 40).double() + 0.5) / 16777216.0
    return (-torch.log(-torch.log(u))).float().to(device)


def sample_tokens(logits: torch.Tensor, temps: torch.Tensor, seeds: torch.Tensor,
                  positions: torch.Tensor) -> torch.Tensor:
    """Gumbel-max sampling (argmax when temperature <= 0); ties -> lowest id."""
    B, V = logits.shape
    out = torch.empty(B, dtype=torch.int32)
    for b in range(B):
        row = logits[b].float().cpu()
        t = float(temps[b])
        if t > 0:
            row = row / t + gumbel_noise(int(seeds[b]), int(positions[b]), V)
        out[b] = int(torch.argmax(row))
    return out.to(logits.device)


def sample_finish(tokens: torch.Tensor, st) -> None:
    """Bookkeeping identical to the finish kernel (st = engine DecodeState)."""
    B = tokens.shape[0]
    eos = set(int(x) for x in st.eos.tolist() if int(x) >= 0)
    for b in range(B):
        if int(st.done[b]):
            continue
        tok = int(tokens[b])
        g = int(st.gen_count[b])
        st.out_tokens[b, g] = tok
        st.gen_count[b] = g + 1
        st.next_ids[b] = tok
        if g + 1 >= int(st.max_new[b]) or tok in eos:
            st.done[b] = 1
        else:
            st.positions[b] += 1


def attention_scale(d: int) -> float:
    return 1.0 / math.sqrt(d)


# ----------------------------------------------------------------- hybrid attention / state-space layers
# A projection result ``u`` is either rows [T, N] in the compute dtype or fp32 split-K slabs [S, T, N]; every consumer
# below takes both.  Recurrent ops take an ops.Segments: the batch as consecutive segments, one per sequence.
def rows32(u: torch.Tensor) -> torch.Tensor:
    return u.float().sum(0) if u.dim() == 3 else u.float()


def embed_pos(ids, positions, table, scale: float, pos_freq) -> torch.Tensor:
    """fp32 rows table[id] * scale + sinusoid(position): entry 2i sin(p f_i), entry 2i + 1 cos(p f_i)."""
    x = table[ids.long().clamp(0, table.shape[0] - 1)].float() * scale
    ang = positions[: ids.numel()].double()[:, None] * pos_freq[None, :]
    pe = torch.stack([ang.sin(), ang.cos()], -1).flatten(1)[:, : x.shape[1]]
    return x + pe.float()


def add_norm32(residual, src, w, eps: float, dtype, width: int) -> torch.Tensor:
    """residual (fp32, in place) += src's first columns; returns rms(residual) * w as ``dtype`` rows, zero-padded to
    ``width``."""
    T, D = residual.shape
    if src is not None:
        residual += rows32(src)[:, :D]
    y = residual * torch.rsqrt(residual.pow(2).mean(-1, keepdim=True) + eps) * w
    out = torch.zeros(T, width, dtype=dtype, device=residual.device)
    out[:, :D] = y.to(dtype)
    return out


def project(x, w) -> torch.Tensor:
    return (x.float() @ w.float().t())[None]


def logits32(x, w) -> torch.Tensor:
    return x.float() @ w.float().t()


def project_glu(x, w_gu, limit: float, alpha: float, shift: float) -> torch.Tensor:
    g, u = split_gate_up(x.float() @ w_gu.float().t())
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(alpha * g) * (u + shift)).to(x.dtype)


def qkv_prep(u, al, bias, q_norm, k_norm, eps: float, out_scale: float, positions, seq_idx, block_tables, kcache,
             vcache, page: int, dtype):
    """Bias, whole-projection q / k norm, query temperature; K / V rows into the paged cache.  Returns (q [T, H * dk]
    with zero-padded heads, gate fp32 [T, H] = out_scale * sigmoid(gate column), or out_scale without a gate)."""
    sp, r = al.spec, rows32(u)
    T, H, G = r.shape[0], sp.heads, sp.kv_heads
    pos, rows = positions[:T].long(), seq_idx[:T].long()

    def part(at, n):
        return r[:, at: at + n] + bias[at: at + n]

    def norm(t, w):
        return t if w is None else t * torch.rsqrt(t.pow(2).mean(-1, keepdim=True) + eps) * w
    q, k, v = norm(part(al.q, H * sp.dim), q_norm), norm(part(al.k, G * sp.dim), k_norm), part(al.v, G * sp.vdim)
    if sp.q_temp is not None:
        coef, every = sp.q_temp
        q = q * (1.0 + coef * torch.log(torch.floor((pos + 1).float() / every) + 1.0))[:, None]
    qo = torch.zeros(T, H, al.dk, dtype=dtype, device=r.device)
    qo[:, :, : sp.dim] = q.view(T, H, sp.dim).to(dtype)
    pages, offs = block_tables[rows, pos // page].long(), pos % page
    kp = torch.zeros(T, G, al.dk, dtype=dtype, device=r.device)
    kp[:, :, : sp.dim] = k.view(T, G, sp.dim).to(dtype)
    vp = torch.zeros(T, G, al.dv, dtype=dtype, device=r.device)
    vp[:, :, : sp.vdim] = v.view(T, G, sp.vdim).to(dtype)
    kcache[pages, :, offs], vcache[pages, :, offs] = kp, vp
    gate = torch.full((T, H), out_scale, dtype=torch.float32, device=r.device)
    if sp.head_gate:
        gate *= torch.sigmoid(r[:, al.g: al.g + H])
    return qo.reshape(T, H * al.dk), gate


def attn_rows(q, kcache, vcache, positions, seq_idx, block_tables, hq: int, hkv: int, pitch: int, page: int,
              scale: float, gate, out) -> None:
    """Every row attends to its sequence's cached keys [0, position]; head h of row t -> out[t, h * pitch :
    (h + 1) * pitch], times gate[t, h]."""
    dk, dv, g = kcache.shape[3], vcache.shape[3], hq // hkv
    for t in range(q.shape[0]):
        n = int(positions[t]) + 1
        pg = block_tables[int(seq_idx[t]), : -(-n // page)].long()
        k = kcache[pg].permute(1, 0, 2, 3).reshape(hkv, -1, dk)[:, :n].float()
        v = vcache[pg].permute(1, 0, 2, 3).reshape(hkv, -1, dv)[:, :n].float()
        s = torch.matmul(q[t].view(hkv, g, dk).float(), k.transpose(1, 2)) * scale
        o = torch.matmul(torch.softmax(s, -1), v).reshape(hq, dv) * gate[t][:, None]
        out[t, : hq * pitch] = o[:, :pitch].reshape(-1).to(out.dtype)


def conv_silu(u, at: int, kernel, bias, state, segs, dtype, gelu=None) -> torch.Tensor:
    """silu(causal per-channel convolution) of columns [at, at + C) of ``u``; ``kernel`` [taps, C] (last tap = current
    token), ``state`` [slots, taps - 1, C] the inputs before each segment (oldest first), updated in place."""
    taps, C = kernel.shape
    r = rows32(u)[:, at: at + C]
    if u.dim() == 3 and dtype != torch.float32:
        r = r.to(dtype).float()  # the short convolution's inputs are rounded alike in both forms of u
    out = torch.empty(r.shape[0], C, dtype=dtype, device=r.device)
    for b, e, slot, pos0 in segs.host():
        h = state[slot] if pos0 > 0 else torch.zeros_like(state[slot])
        x = torch.cat([h[: taps - 1], r[b:e]])
        y = sum(kernel[j] * x[j: j + e - b] for j in range(taps)) + bias
        out[b:e] = (y * torch.sigmoid(y)).to(dtype)
        if taps > 1:
            state[slot] = x[-(taps - 1):]
    return out


def ssm_scan(xbc, u, dt_at: int, dt_bias, a_neg, d_skip, state, segs, heads: int, vdim: int, n_state: int, groups: int):
    """y_t = S_t^T C_t + D x_t with S_t = exp(a dt) S_(t-1) + dt B_t x_t^T per head; ``state`` [slots, heads, vdim, N']
    (S^T, fp32) is carried in place.  Returns fp32 [T, heads * vdim]."""
    T = xbc.shape[0]
    f = xbc.float()
    inner, gn = heads * vdim, groups * n_state
    x = f[:, :inner].view(T, heads, vdim)
    rep = heads // groups
    B = f[:, inner: inner + gn].view(T, groups, n_state).repeat_interleave(rep, 1)
    C = f[:, inner + gn: inner + 2 * gn].view(T, groups, n_state).repeat_interleave(rep, 1)
    dt = torch.nn.functional.softplus(rows32(u)[:, dt_at: dt_at + heads] + dt_bias, threshold=30.0)
    y = torch.empty(T, heads, vdim, dtype=torch.float32, device=f.device)
    for b, e, slot, pos0 in segs.host():
        S = state[slot, :, :, :n_state].clone() if pos0 > 0 else torch.zeros(heads, vdim, n_state, device=f.device)
        for t in range(b, e):
            S = torch.exp(a_neg * dt[t])[:, None, None] * S + (dt[t][:, None] * x[t])[:, :, None] * B[t][:, None, :]
            y[t] = (S * C[t][:, None, :]).sum(-1) + d_skip[:, None] * x[t]
        state[slot, :, :, :n_state] = S
    return y.view(T, inner)


def gated_norm(y, u, z_at: int, w, norm_groups: int, eps: float, out_scale: float, out, col: int) -> None:
    """out[:, col : col + inner] = out_scale * w * grouped RMS norm of y * silu(z); zeros in the columns after it."""
    T, n = y.shape
    z = rows32(u)[:, z_at: z_at + n]
    v = (y.float() * z * torch.sigmoid(z)).view(T, norm_groups, -1)
    v = v * torch.rsqrt(v.pow(2).mean(-1, keepdim=True) + eps)
    out[:, col: col + n] = (v.reshape(T, n) * w * out_scale).to(out.dtype)
    out[:, col + n:] = 0


# ----------------------------------------------------------------- bigram embedding, gelu, rotation
def embed_bigram(ids, segs, table, bigram, scale: float, mul_prev: int, mul_cur: int, w, eps: float, last) -> torch.Tensor:
    """fp32 rows rms(table[id] * scale + bigram[pair]) * w.  ``last`` [slots]: the token before each segment's first
    (a segment at position 0 has none: the table's last row), replaced by the segment's last token."""
    buckets = bigram.shape[0] - 1
    tok = ids.long()
    row = torch.empty_like(tok)
    for b, e, slot, pos0 in segs.host():
        prev = torch.cat([last[slot: slot + 1].long(), tok[b: e - 1]])
        row[b:e] = (prev * mul_prev + tok[b:e] * mul_cur) % buckets
        if pos0 == 0:
            row[b] = buckets
        last[slot] = ids[e - 1]
    x = table[tok.clamp(0, table.shape[0] - 1)].float() * scale + bigram[row].float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w


def project_gelu(x, w, n: int, out, col: int, cols: int):
    """The first ``n`` rows of ``w`` as project(); gelu of the next ``cols`` into out[:, col : col + cols]."""
    u = x.float() @ w[: n + cols].float().t()
    out[:, col: col + cols] = torch.nn.functional.gelu(u[:, n:], approximate="tanh").to(out.dtype)
    return u[None, :, :n].contiguous(), None


def yarn_inv_freq(dims: int, base: float, yarn=None) -> torch.Tensor:
    """Rotary frequencies (float64) of config.RotarySpec."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = base ** (-2.0 * i / dims)
    if yarn is None:
        return f

    def dim_of(turns: float) -> float:
        return dims * math.log(yarn.original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(dim_of(yarn.fast)), 0), min(math.ceil(dim_of(yarn.slow)), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / yarn.factor * ramp + f * (1.0 - ramp)


def rotary_table(max_pos: int, rot, device=None) -> torch.Tensor:
    """[max_pos, dims / 2, 2] fp32 (cosine, sine) of config.RotarySpec, the angles in float64."""
    s = rot.scaling
    m = 1.0 if s is None else 0.1 * math.log(s.factor) + 1.0
    ang = torch.outer(torch.arange(max_pos, dtype=torch.float64), yarn_inv_freq(rot.dims, rot.base, s))
    return (torch.stack([ang.cos(), ang.sin()], -1) * m).float().contiguous().to(device)


def rotate_half(x: torch.Tensor, cs: torch.Tensor) -> torch.Tensor:
    """Rows x [..., dims] with their (cosine, sine) rows cs [..., dims / 2, 2]."""
    h = x.shape[-1] // 2
    u, v, c, s = x[..., :h], x[..., h:], cs[..., 0], cs[..., 1]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


# ----------------------------------------------------------------- latent attention (``m``: engine.mixers.LatentMixer)
def latent_prep(u, m, dq_norm, dkv_norm, eps: float, cs, positions, seq_idx, block_tables, cache, page: int, dtype,
                gelu=None):
    """Normed query latents [T, m.cq] (zero-padded); for a layer with its own latents, the row [normed latent | rotated
    key part] of every token into the paged cache."""
    sp, r = m.spec, rows32(u)
    T = r.shape[0]

    def norm(t, w):
        return t * torch.rsqrt(t.pow(2).mean(-1, keepdim=True) + eps) * w
    out = torch.zeros(T, m.cq, dtype=dtype, device=r.device)
    out[:, : sp.q_rank] = norm(r[:, m.dq: m.dq + sp.q_rank], dq_norm).to(dtype)
    if dkv_norm is not None:
        pos = positions[:T].long()
        row = torch.zeros(T, m.row, dtype=dtype, device=r.device)
        row[:, : sp.kv_rank] = norm(r[:, m.dkv: m.dkv + sp.kv_rank], dkv_norm).to(dtype)
        row[:, m.rank8: m.rank8 + sp.rot_dim] = rotate_half(r[:, m.dkr: m.dkr + sp.rot_dim], cs[pos]).to(dtype)
        cache[block_tables[seq_idx[:T].long(), pos // page].long(), 0, pos % page] = row
    return out


def latent_absorb(q, n: int, m, w_uk, cs, positions, dtype) -> torch.Tensor:
    """Queries of the first ``n`` rows against cached rows: [n, H * row], per head [W_uk^T q | rotated part]."""
    sp = m.spec
    r = rows32(q)[:n, : sp.heads * m.qw].view(n, sp.heads, m.qw).to(dtype).float()
    out = torch.zeros(n, sp.heads, m.row, dtype=dtype, device=r.device)
    out[:, :, : m.rank8] = torch.einsum("thd,hrd->thr", r[:, :, : sp.dim], w_uk[:, :, : sp.dim].float()).to(dtype)
    rot = r[:, :, m.dim8: m.dim8 + sp.rot_dim]
    out[:, :, m.rank8: m.rank8 + sp.rot_dim] = rotate_half(rot, cs[positions[:n].long()][:, None]).to(dtype)
    return out.view(n, -1)


def latent_rows(q, cache, positions, seq_idx, block_tables, heads: int, rank: int, page: int, scale: float):
    """Attention of absorbed query rows over the cached rows: weighted sums of latents [T, H * rank]."""
    T, row = q.shape[0], cache.shape[3]
    out = torch.empty(T, heads, rank, dtype=q.dtype, device=q.device)
    for t in range(T):
        n = int(positions[t]) + 1
        c = cache[block_tables[int(seq_idx[t]), : -(-n // page)].long(), 0].reshape(-1, row)[:n].float()
        p = torch.softmax((q[t].view(heads, row).float() @ c.t()) * scale, -1)
        out[t] = (p @ c[:, :rank]).to(q.dtype)
    return out.view(T, -1)


def latent_out(o, m, w_uv, a, col: int) -> None:
    """a[:, col : col + H * vp] = per head W_uv (weighted latent sum)."""
    H = m.spec.heads
    y = torch.einsum("thr,hnr->thn", o.view(o.shape[0], H, m.rank8).float(), w_uv[:, :, : m.rank8].float())
    a[:, col: col + H * m.vp] = y.reshape(o.shape[0], -1).to(a.dtype)


# ----------------------------------------------------------------- gated delta rule (``m``: engine.mixers.DeltaMixer)
def delta_mix(x, u, m, a_neg, dt_bias, norm, eps: float, state, segs, a) -> None:
    """Unit queries and keys, step sizes and decays, the recurrence with ``state`` [slots, heads, vdim, dim'] (S^T, fp32)
    carried in place, and the gated head-wise output norm into a[:, m.col : m.col + m.width]."""
    sp = m.spec
    T, H, G, d, dv = x.shape[0], sp.heads, sp.kv_heads, sp.dim, sp.vdim
    f, r = x.float(), rows32(u)

    def unit(t):
        return t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) + 1e-6)
    q = (unit(f[:, : G * d].view(T, G, d)) * d ** -0.5).repeat_interleave(H // G, 1)
    k = unit(f[:, m.xk: m.xk + G * d].view(T, G, d)).repeat_interleave(H // G, 1)
    v = f[:, m.xv: m.xv + H * dv].view(T, H, dv)
    beta = torch.sigmoid(r[:, m.b: m.b + H])
    g = torch.exp(a_neg * torch.nn.functional.softplus(r[:, m.a: m.a + H] + dt_bias, threshold=30.0))
    y = torch.empty(T, H, dv, dtype=torch.float32, device=f.device)
    for b, e, slot, pos0 in segs.host():
        S = state[slot, :, :, :d].clone() if pos0 > 0 else torch.zeros(H, dv, d, device=f.device)
        for t in range(b, e):
            S = g[t][:, None, None] * S
            w = beta[t][:, None] * (v[t] - (S * k[t][:, None, :]).sum(-1))
            S = S + w[:, :, None] * k[t][:, None, :]
            y[t] = (S * q[t][:, None, :]).sum(-1)
        state[slot, :, :, :d] = S
    z = r[:, m.g: m.g + H * dv].view(T, H, dv)
    y = y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + eps) * norm * (z * torch.sigmoid(z))
    a[:, m.col: m.col + m.width] = 0
    a[:, m.col: m.col + H * dv] = y.reshape(T, H * dv).to(a.dtype)
