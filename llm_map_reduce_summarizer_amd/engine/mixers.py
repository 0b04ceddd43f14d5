"""Mixers of the hybrid decoders (engine/hybrid.py): grouped-query attention, Mamba-2 state-space mixer, latent attention
and the gated delta rule.

A mixer owns a range of columns of its layer's fused input projection and of its output rows:

    columns(take)      reserve projection columns; ``width`` is what it writes into the joint output rows
    load(...)          its weights, asked for by checkpoint name
    cache_shape / state_shape     what a sequence holds for it: paged rows, recurrent state
    run(i, u, a, b, kv, eps, gelu)      projection rows u -> a[:, col : col + width]; ``gelu``: the layer's pending
                                  feed-forward columns (ops.project_gelu), for mixers that take them along (takes_gelu)

``b`` is the batch: ``n_decode`` leading single tokens (decode kernels), prompt portions behind them.
"""

from __future__ import annotations

from types import SimpleNamespace
from typing import Callable, Dict, Optional, Tuple

import torch

from .. import ops
from .config import AttnSpec, DeltaSpec, LatentSpec, SSMSpec

MFMA_HEAD = 128  # padded head width of the grouped-query MFMA attention kernels; wider heads run the row kernel


def up(n: int, m: int) -> int:
    return -(-n // m) * m


class Loader:
    """Checkpoint access and weight placement of one model: zero-padded matrices of the compute dtype, fp32 vectors."""

    def __init__(self, get: Callable, device: torch.device, dtype: torch.dtype):
        self.get, self.device, self.dtype = get, device, dtype

    def mat(self, *shape: int) -> torch.Tensor:
        return torch.zeros(*shape, dtype=self.dtype, device=self.device)

    def vec(self, name: str, n: int, offset: float = 0.0) -> torch.Tensor:
        return (self.get(name, (n,)).to(self.device).float() + offset).contiguous()

    def fetch(self, name: str, *shape: int) -> torch.Tensor:
        return self.get(name, shape).to(device=self.device, dtype=self.dtype)

    def put(self, dst: torch.Tensor, r0: int, c0: int, t: torch.Tensor) -> None:
        dst[r0:r0 + t.shape[0], c0:c0 + t.shape[1]] = t.to(device=self.device, dtype=self.dtype)


class Mixer:
    width = 0          # columns of the joint output rows
    col = 0            # first of them
    scale = 1.0        # factor on this mixer's share of the layer's sum
    takes_gelu = False

    def __init__(self):
        self.w = SimpleNamespace()

    def cache_shape(self) -> Optional[Tuple[int, int, int]]:
        return None

    def state_shape(self) -> Optional[Tuple[int, int, int, int, int]]:
        return None

    def decode_workspace(self, B: int, max_ctx: int, device) -> Optional[Tuple[object, object]]:
        """(key, split-K buffers) of the decode kernel, shared by the mixers of the same key."""
        return None

    def pass_items(self, lens) -> Optional[Tuple[object, object]]:
        """(key, work list) of the prompt-portion kernel."""
        return None


class AttnMixer(Mixer):
    """Grouped-query attention (AttnSpec)."""

    def __init__(self, spec: AttnSpec, device: torch.device, dtype: torch.dtype, scale: float):
        super().__init__()
        a = self.spec = spec
        self.dtype, self.scale = dtype, scale
        # 16-bit heads of at most MFMA_HEAD: the MFMA prefill / decode kernels
        self.mfma = device.type == "cuda" and dtype == torch.bfloat16 and max(a.dim, a.vdim) <= MFMA_HEAD \
            and a.heads // a.kv_heads <= 64
        self.dk = MFMA_HEAD if self.mfma else up(a.dim, 8)   # cached key width (also the pitch of the q rows' heads)
        self.dv = MFMA_HEAD if self.mfma else up(a.vdim, 8)  # cached value width
        self.vp = up(a.vdim, 8)                              # output pitch of one head
        self.width = a.heads * self.vp

    def columns(self, take) -> None:
        a = self.spec
        self.q, self.k = take(a.heads * a.dim), take(a.kv_heads * a.dim)
        self.v, self.g = take(a.kv_heads * a.vdim), take(a.heads if a.head_gate else 0)

    def load(self, ld: Loader, m: str, w_in, w_o, hidden: int) -> None:
        a, w = self.spec, self.w
        qn, kn, vn = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim
        for name, at, n in (("q", self.q, qn), ("k", self.k, kn), ("v", self.v, vn)):
            ld.put(w_in, at, 0, ld.get(m + name, (n, hidden)))
        w.qkv_bias = torch.zeros(w_in.shape[0], dtype=torch.float32, device=ld.device)  # at the projection's columns
        if a.bias:
            for name, at, n in (("q.b", self.q, qn), ("k.b", self.k, kn), ("v.b", self.v, vn)):
                w.qkv_bias[at:at + n] = ld.vec(m + name, n)
        w.q_norm = ld.vec(m + "q.norm", qn) if a.qk_norm else None
        w.k_norm = ld.vec(m + "k.norm", kn) if a.qk_norm else None
        if a.head_gate:
            ld.put(w_in, self.g, 0, ld.get(m + "g", (a.heads, hidden)))
        wo = ld.get(m + "o", (hidden, a.heads * a.vdim))
        for h in range(a.heads):
            ld.put(w_o, 0, self.col + h * self.vp, wo[:, h * a.vdim:(h + 1) * a.vdim])

    def cache_shape(self):
        return (self.spec.kv_heads, self.dk, self.dv)

    def decode_workspace(self, B, max_ctx, device):
        if not self.mfma:
            return None
        key = (self.spec.heads, self.spec.kv_heads)
        return key, lambda: ops.decode_workspace(B, key[0], key[1], MFMA_HEAD, max_ctx, device)

    def pass_items(self, lens):
        if not self.mfma:
            return None
        r = self.spec.heads // self.spec.kv_heads
        return r, lambda: ops.prefill_items(lens, r)

    def run(self, i, u, a, b, kv, eps, gelu=None) -> None:
        sp, w, page, T = self.spec, self.w, kv.page, a.shape[0]
        kc, vc = kv.k[i], kv.v[i]
        q, gate = ops.qkv_prep(u, self, w.qkv_bias, w.q_norm, w.k_norm, eps, self.scale, b.positions, b.seq_idx,
                               b.tables, kc, vc, page, self.dtype)
        if not self.mfma:
            ops.attn_rows(q, kc, vc, b.positions, b.seq_idx, b.tables, sp.heads, sp.kv_heads, self.vp, page, sp.scale,
                          gate, a)
            return
        nd = b.n_decode
        if nd:
            ops.attn_decode(q[:nd], kc, vc, b.decode_tables, b.positions, sp.heads, sp.kv_heads, MFMA_HEAD, page,
                            sp.scale, out=a[:nd], workspace=b.workspace.get((sp.heads, sp.kv_heads)), gate=gate[:nd],
                            pitch=self.vp)
        if nd < T:
            ops.attn_prefill(q[nd:], b.cu_portions, sp.heads, sp.kv_heads, MFMA_HEAD, sp.scale, out=a[nd:],
                             paged=b.paged.layer(kc, vc), seqlens=b.portion_lens,
                             items=b.items[sp.heads // sp.kv_heads], gate=gate[nd:], pitch=self.vp)


class SSMMixer(Mixer):
    """Mamba-2 (SSMSpec)."""

    takes_gelu = True

    def __init__(self, spec: SSMSpec, device: torch.device, dtype: torch.dtype, scale: float):
        super().__init__()
        self.spec, self.dtype, self.scale = spec, dtype, scale
        self.width = spec.inner

    def columns(self, take) -> None:
        s = self.spec
        self.z, self.xbc, self.dt = take(s.inner), take(s.channels), take(s.heads)

    def load(self, ld: Loader, m: str, w_in, w_o, hidden: int) -> None:
        s, w = self.spec, self.w
        win = ld.get(m + "in", (s.in_rows, hidden))
        ld.put(w_in, self.z, 0, win[:s.inner])
        ld.put(w_in, self.xbc, 0, win[s.inner:s.inner + s.channels])
        ld.put(w_in, self.dt, 0, win[s.inner + s.channels:])
        cp = up(s.channels, 8)  # the convolution runs on whole groups of 8 channels
        w.conv = torch.zeros(s.conv, cp, dtype=torch.float32, device=ld.device)
        w.conv[:, :s.channels] = ld.get(m + "conv", (s.channels, s.conv)).to(ld.device).float().t()
        w.conv_b = torch.zeros(cp, dtype=torch.float32, device=ld.device)
        w.conv_b[:s.channels] = ld.vec(m + "conv.b", s.channels)
        w.dt_bias = ld.vec(m + "dt_bias", s.heads)
        w.a_neg = -torch.exp(ld.vec(m + "A_log", s.heads))
        w.d_skip = ld.vec(m + "D", s.heads)
        w.ssm_norm = ld.vec(m + "norm", s.inner)
        ld.put(w_o, 0, self.col, ld.get(m + "o", (hidden, s.inner)))

    def state_shape(self):
        s = self.spec
        return (up(s.channels, 8), s.conv, s.heads, s.vdim, s.state)

    def run(self, i, u, a, b, kv, eps, gelu=None) -> None:
        s, w, st = self.spec, self.w, kv.state
        xbc = ops.conv_silu(u, self.xbc, w.conv, w.conv_b, st.conv[i], b.segs, self.dtype, gelu)
        y = ops.ssm_scan(xbc, u, self.dt, w.dt_bias, w.a_neg, w.d_skip, st.ssm[i], b.segs, s.heads, s.vdim, s.state,
                         s.groups)
        ops.gated_norm(y, u, self.z, w.ssm_norm, s.norm_groups, eps, self.scale, a, self.col)


class LatentMixer(Mixer):
    """Latent attention (LatentSpec).  A cached row is [latent | rotated key part], each padded to 8 columns.

    Prompt portions: the latents of each sequence's whole context are gathered from the cache and expanded to every
    head's unrotated keys and values (one product), and flash attention runs on [expanded key | shared rotated part].
    Decoded tokens, 32-bit models and head sizes outside the MFMA kernels: the key expansion is absorbed into the
    query, so scores and value sums run on the cached rows themselves, and the value expansion follows."""

    takes_gelu = True

    def __init__(self, spec: LatentSpec, device: torch.device, dtype: torch.dtype):
        super().__init__()
        s = self.spec = spec
        self.dtype = dtype
        self.dim8, self.rot8, self.rank8 = up(s.dim, 8), up(s.rot_dim, 8), up(s.kv_rank, 8)
        self.qw = self.dim8 + self.rot8       # one head of the query rows
        self.row = self.rank8 + self.rot8     # one cached row
        self.vp = up(s.vdim, 16)              # output pitch of one head
        self.cq = up(s.q_rank, 128)           # normed query latent rows
        self.width = s.heads * self.vp
        on = device.type == "cuda" and dtype == torch.bfloat16
        self.flash = on and ops.latent_prefill_ok(self.dim8, self.rot8, self.vp)
        self.mfma = on and ops.latent_decode_ok(self.rank8, self.row)
        # expanded rows: unrotated keys of all heads, then their values
        self.kv_v = s.heads * self.dim8
        self.kv_n = up(self.kv_v + s.heads * self.vp, 16)
        self.lat_k = up(s.kv_rank, 64)                       # depth of the expansion product
        self.lat = max(self.row, self.lat_k)                 # gathered row: the cached one, zeros behind it

    def columns(self, take) -> None:
        s = self.spec
        self.dq = take(s.q_rank)
        self.dkv = take(s.kv_rank) if s.kv_from is None else -1
        self.dkr = take(s.rot_dim) if s.kv_from is None else -1

    def load(self, ld: Loader, m: str, w_in, w_o, hidden: int) -> None:
        s, w, H = self.spec, self.w, self.spec.heads
        ld.put(w_in, self.dq, 0, ld.get(m + "dq", (s.q_rank, hidden)))
        w.dq_norm = ld.vec(m + "dq.norm", s.q_rank)
        w.dkv_norm = None
        if s.kv_from is None:
            dkv = ld.get(m + "dkv", (s.kv_rank + s.rot_dim, hidden))
            ld.put(w_in, self.dkv, 0, dkv[:s.kv_rank])
            ld.put(w_in, self.dkr, 0, dkv[s.kv_rank:])
            w.dkv_norm = ld.vec(m + "dkv.norm", s.kv_rank)
        uq = ld.fetch(m + "uq", H * (s.dim + s.rot_dim), s.q_rank).view(H, s.dim + s.rot_dim, s.q_rank)
        w.w_uq = ld.mat(up(H * self.qw, 128), self.cq)
        t = w.w_uq[:H * self.qw].view(H, self.qw, self.cq)
        t[:, :s.dim, :s.q_rank] = uq[:, :s.dim]
        t[:, self.dim8:self.dim8 + s.rot_dim, :s.q_rank] = uq[:, s.dim:]
        uk = ld.fetch(m + "uk", H * s.dim, s.kv_rank).view(H, s.dim, s.kv_rank)
        uv = ld.fetch(m + "uv", H * s.vdim, s.kv_rank).view(H, s.vdim, s.kv_rank)
        w.w_uk = ld.mat(H, self.rank8, up(s.dim, 32))     # per head: query part -> latent space
        w.w_uk[:, :s.kv_rank, :s.dim] = uk.transpose(1, 2)
        w.w_uv = ld.mat(H, self.vp, up(s.kv_rank, 32))    # per head: latent space -> value
        w.w_uv[:, :s.vdim, :s.kv_rank] = uv
        if self.flash:
            w.w_kv = ld.mat(self.kv_n, self.lat_k)        # latents -> all heads' keys and values
            w.w_kv[:self.kv_v].view(H, self.dim8, self.lat_k)[:, :s.dim, :s.kv_rank] = uk
            w.w_kv[self.kv_v:self.kv_v + H * self.vp].view(H, self.vp, self.lat_k)[:, :s.vdim, :s.kv_rank] = uv
        wo = ld.get(m + "o", (hidden, H * s.vdim))
        for h in range(H):
            ld.put(w_o, 0, self.col + h * self.vp, wo[:, h * s.vdim:(h + 1) * s.vdim])

    def cache_shape(self):
        return (1, self.row, 0) if self.spec.kv_from is None else None

    def decode_workspace(self, B, max_ctx, device):
        if not self.mfma:
            return None
        H, rank = self.spec.heads, self.rank8
        return ("latent", H, rank), lambda: ops.latent_workspace(B, H, rank, max_ctx, device)

    def pass_items(self, lens):
        if not self.flash:
            return None
        rows = ops.latent_block_rows(self.qw, self.vp)
        return ("latent", rows), lambda: ops.latent_items(lens, rows)

    def run(self, i, u, a, b, kv, eps, gelu=None) -> None:
        s, w, page, T = self.spec, self.w, kv.page, a.shape[0]
        src = i if s.kv_from is None else s.kv_from
        cache, cs = kv.k[src], b.rotary[s.rot]
        cq = ops.latent_prep(u, self, w.dq_norm, w.dkv_norm, eps, cs, b.positions, b.seq_idx, b.tables, cache, page,
                             self.dtype, gelu)
        q = ops.project(cq, w.w_uq, "qkv")
        nd = b.n_decode if self.flash else T
        if nd:
            qa = ops.latent_absorb(q, nd, self, w.w_uk, cs, b.positions, self.dtype)
            if self.mfma and b.n_decode:
                n = b.n_decode
                ws = b.workspace.get(("latent", s.heads, self.rank8))
                parts = ops.latent_decode(qa[:n], cache, b.decode_tables, b.positions, s.heads, self.rank8, page,
                                          s.scale, ws)
                ops.latent_out_parts(parts, self, w.w_uv, a[:n], self.col)
            n = b.n_decode if self.mfma else 0
            if n < nd:
                o = ops.latent_rows(qa[n:], cache, b.positions[n:nd], b.seq_idx[n:nd], b.tables, s.heads, self.rank8,
                                    page, s.scale)
                ops.latent_out(o, self, w.w_uv, a[n:nd], self.col)
        if nd < T:
            ctx = b.context()
            key = ("latents", src)
            if key not in b.shared:
                b.shared[key] = ops.latent_gather(cache, ctx, b.tables, self.lat, page)
            lat = b.shared[key]
            qr = ops.latent_rope(q, nd, self, cs, b.positions)
            kvx = ops.latent_expand(lat, w.w_kv)
            ops.latent_prefill(qr, kvx, lat, ctx, self, b.cu_portions, b.portion_lens,
                               b.items[("latent", ops.latent_block_rows(self.qw, self.vp))], s.scale, a[nd:], self.col)


class DeltaMixer(Mixer):
    """Gated delta rule (DeltaSpec).  The short convolutions of q, k and v run as one over adjacent columns."""

    takes_gelu = True

    def __init__(self, spec: DeltaSpec, device: torch.device, dtype: torch.dtype):
        super().__init__()
        self.spec, self.dtype = spec, dtype
        self.width = up(spec.inner, 16)
        if device.type == "cuda" and not ops.delta_ok(spec.vdim, spec.dim):
            raise ValueError("delta heads of %d x %d are wider than the kernels take" % (spec.dim, spec.vdim))

    def columns(self, take) -> None:
        s = self.spec
        self.q, self.k, self.v = take(s.kv_heads * s.dim), take(s.kv_heads * s.dim), take(s.inner)
        self.channels = self.v + up(s.inner, 8) - self.q
        self.xk, self.xv = self.k - self.q, self.v - self.q  # first columns of k and v in the convolution's output
        self.g, self.b, self.a = take(s.inner), take(s.heads), take(s.heads)

    def load(self, ld: Loader, m: str, w_in, w_o, hidden: int) -> None:
        s, w = self.spec, self.w
        w.conv = torch.zeros(s.conv, self.channels, dtype=torch.float32, device=ld.device)
        w.conv_b = torch.zeros(self.channels, dtype=torch.float32, device=ld.device)
        for name, at, n in (("q", self.q, s.kv_heads * s.dim), ("k", self.k, s.kv_heads * s.dim), ("v", self.v, s.inner)):
            ld.put(w_in, at, 0, ld.get(m + name, (n, hidden)))
            w.conv[:, at - self.q: at - self.q + n] = ld.get(m + name + ".conv", (n, s.conv)).to(ld.device).float().t()
        ld.put(w_in, self.g, 0, ld.get(m + "g", (s.inner, hidden)))
        ld.put(w_in, self.b, 0, ld.get(m + "b", (s.heads, hidden)))
        ld.put(w_in, self.a, 0, ld.get(m + "a", (s.heads, hidden)))
        w.a_neg = -torch.exp(ld.vec(m + "A_log", s.heads))
        w.dt_bias = ld.vec(m + "dt_bias", s.heads)
        w.norm = ld.vec(m + "norm", s.vdim)
        ld.put(w_o, 0, self.col, ld.get(m + "o", (hidden, s.inner)))

    def state_shape(self):
        s = self.spec
        return (self.channels, s.conv, s.heads, s.vdim, s.dim)

    def run(self, i, u, a, b, kv, eps, gelu=None) -> None:
        w, st = self.w, kv.state
        x = ops.conv_silu(u, self.q, w.conv, w.conv_b, st.conv[i], b.segs, self.dtype, gelu)
        ops.delta_mix(x, u, self, w.a_neg, w.dt_bias, w.norm, eps, st.ssm[i], b.segs, a)


def workspaces(mixers, B: int, max_ctx: int, device) -> Dict[object, object]:
    out: Dict[object, object] = {}
    for m in mixers:
        e = m.decode_workspace(B, max_ctx, device)
        if e is not None and e[0] not in out:
            out[e[0]] = e[1]()
    return out


def work_items(mixers, lens, device) -> Dict[object, object]:
    out: Dict[object, object] = {}
    for m in mixers if lens else ():
        e = m.pass_items(lens)
        if e is not None and e[0] not in out:
            out[e[0]] = e[1]().to(device, non_blocking=True)
    return out
