"""Forward pass of the decoders whose layers are listed one by one (config.HybridConfig: the Merulorn and Muzozen
designs).  The mixers are in engine/mixers.py.

The residual stream is fp32.  One layer, in every phase (prompt portions, decoded tokens, or both in one batch):

    x  = norm(residual)                       x rows in the compute dtype, gain (offset + w)
    u  = x @ w_in^T                           ONE product for the input columns of all mixers
    mixers: u -> a[:, columns of the mixer]   paged cache, recurrent state and conv taps in the request's state slot
    residual += a @ w_o^T                     w_o = the mixers' output projections side by side, so the sum of the mixers
                                              is part of the product; added in fp32 by the next norm kernel

Feed-forward behind the mixers (Merulorn): norm, w_gu ([8 gate | 8 up] rows) -> clamped GLU -> w_down, added the same
way.  Feed-forward beside them (Muzozen): its up rows follow the mixers' columns in w_in, gelu writes a's last columns,
and w_down stands beside the mixers' output projections in w_o -- one product in, one product out per layer.

Projections with few rows leave fp32 split-K slabs that their consumer kernel sums (ops.project); with many rows
they are 16-bit rows of the MFMA GEMM.  In 32-bit mode everything is fp32 (ops.project -> the fp32 MFMA GEMM).

Sizes are free: weight rows / columns are zero-padded at load to what the GEMM kernels take (rows to a multiple of
16, products to a multiple of 128), heads to the cache's key / value widths.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from types import SimpleNamespace
from typing import Callable, Dict, List, Optional, Sequence, Tuple

import torch

from .. import ops
from ..ops.reference import interleave_gate_up, rotary_table
from .config import GLUSpec, HybridConfig, LayerSpec
from .mixers import AttnMixer, DeltaMixer, LatentMixer, Loader, Mixer, SSMMixer, up, work_items, workspaces
from .model import _randn


@dataclass
class HybridLayer:
    spec: LayerSpec
    attn: Optional[AttnMixer] = None
    ssm: Optional[SSMMixer] = None
    latent: Optional[LatentMixer] = None
    delta: Optional[DeltaMixer] = None
    n_mix: int = 0   # rows of w_in that are the mixers' (padded); a parallel feed-forward's rows follow them
    n_in: int = 0
    ff_col: int = 0  # parallel feed-forward: its columns of the joint output rows
    ff: int = 0
    k_mix: int = 0   # columns of the joint output rows that the mixers write
    k_out: int = 0   # columns of the joint output rows (padded)
    w: SimpleNamespace = field(default_factory=SimpleNamespace)

    @property
    def mixers(self) -> List[Mixer]:
        return [m for m in (self.attn, self.ssm, self.latent, self.delta) if m is not None]


class HybridModel:
    recurrent = True
    float32_kernels = True  # dtype float32 runs on the GPU too

    def __init__(self, cfg: HybridConfig, device: torch.device, dtype: torch.dtype = torch.bfloat16, seed: int = 0,
                 tp_rank: int = 0, tp_size: int = 1, tp_group=None, weight_dtype: str = "bf16",
                 weights_path: Optional[str] = None):
        if tp_size != 1:
            raise ValueError("%s: hybrid models are not sharded (TP=1 only)" % cfg.name)
        if weight_dtype != "bf16":
            raise ValueError("%s: hybrid models take 16-bit (or, with dtype float32, 32-bit) weights" % cfg.name)
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("hybrid models run in bfloat16 or float32")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.weight_dtype = weight_dtype
        self.custom_ar = None
        self.tp_sampling = self.sequence_parallel = self.emulate_tp_reduce = False
        self.layer_hook: Optional[Callable[[int, torch.Tensor], None]] = None  # (layer, residual) after every layer
        self.kp = up(cfg.hidden, 128)
        self.layers = [self._layout(la) for la in cfg.layers]
        if weights_path:
            from .weights import checkpoint_reader
            self._fill(checkpoint_reader(weights_path))
        else:
            self._fill(self._random(seed))
        if cfg.pos_base is not None:
            self.pos_freq = (cfg.pos_base ** (-torch.arange(0, up(cfg.hidden, 2), 2, dtype=torch.float64)
                                              / cfg.hidden)).to(self.device)
        # one table of (cosine, sine) per kind of rotation
        self.rotary = {rot: rotary_table(cfg.max_position, rot, self.device)
                       for rot in {la.spec.latent.rot for la in self.layers if la.latent is not None}}

    # ------------------------------------------------------------------ layouts and weights
    def _layout(self, la: LayerSpec) -> HybridLayer:
        """Column offsets of the fused projections; every section starts at a multiple of 8 columns."""
        out = HybridLayer(la)
        n = 0

        def take(rows: int) -> int:
            nonlocal n
            at, n = n, up(n + rows, 8)
            return at
        if la.attn is not None:
            out.attn = AttnMixer(la.attn, self.device, self.dtype, la.attn_scale)
        if la.ssm is not None:
            out.ssm = SSMMixer(la.ssm, self.device, self.dtype, la.ssm_scale)
        if la.latent is not None:
            out.latent = LatentMixer(la.latent, self.device, self.dtype)
        if la.delta is not None:
            out.delta = DeltaMixer(la.delta, self.device, self.dtype)
        for m in out.mixers:
            m.columns(take)
            m.col = out.k_mix
            out.k_mix += m.width
        out.n_in = out.n_mix = up(n, 128)
        out.k_out = up(out.k_mix, 128)
        if la.parallel and la.mlp is not None:
            out.ff_col = out.k_mix
            out.k_out = up(out.k_mix + la.mlp.ff, 128)
            out.ff = out.k_out - out.ff_col
            out.n_in = up(out.n_mix + out.ff, 128)
        return out

    def _random(self, seed: int):
        """get(name, shape) of seeded random weights in checkpoint form (norm weights around their neutral value)."""
        off = 1.0 - self.cfg.norm_offset

        def get(name, shape):
            leaf = name.rsplit(".", 1)[-1]
            std, mean = self.cfg.init_std, 0.0
            if leaf in ("norm1", "norm2") or name in ("final.norm", "embed.norm"):
                std, mean = 0.1, off
            elif leaf == "norm" or leaf == "D":
                std, mean = 0.1, 1.0
            elif leaf in ("conv", "A_log"):
                std = 0.5
            elif leaf == "dt_bias":
                std, mean = 0.5, -3.0
            elif leaf in ("embed", "bigram"):
                std = 1.0 / max(1.0, self.cfg.embed_scale)
            t = _randn(shape, std, seed, name, self.device, torch.bfloat16)
            return t + mean if mean else t
        return get

    def _fill(self, get) -> None:
        c, H = self.cfg, self.cfg.hidden
        ld = Loader(get, self.device, self.dtype)
        mat, vec, put = ld.mat, ld.vec, ld.put
        self.embed = ld.fetch("embed", c.vocab_size, H).contiguous()
        self.bigram = self.embed_norm = None
        if c.bigram is not None:
            self.bigram = ld.fetch("bigram", c.bigram.buckets + 1, H).contiguous()
            self.embed_norm = vec("embed.norm", H, c.norm_offset)
        self.final_norm = vec("final.norm", H, c.norm_offset)
        self.lm_head = mat(up(c.vocab_size, 128), self.kp)
        put(self.lm_head, 0, 0, get("head", (c.vocab_size, H)))
        for i, la in enumerate(self.layers):
            p, w, spec = "l%d." % i, la.w, la.spec
            w.norm1 = vec(p + "norm1", H, c.norm_offset)
            w.w_in = mat(la.n_in, self.kp)
            w.w_o = mat(up(H, 16), la.k_out)
            side = {id(la.attn): "left.", id(la.ssm): "right."} if len(la.mixers) > 1 else {}
            for m in la.mixers:
                m.load(ld, p + "mix." + side.get(id(m), ""), w.w_in, w.w_o, H)
            if isinstance(spec.mlp, GLUSpec):
                f, fp = spec.mlp.ff, up(spec.mlp.ff, 128)
                w.norm2 = vec(p + "norm2", H, c.norm_offset)
                g, u = mat(fp, self.kp), mat(fp, self.kp)
                put(g, 0, 0, get(p + "mlp.gate", (f, H)))
                put(u, 0, 0, get(p + "mlp.up", (f, H)))
                w.w_gu = interleave_gate_up(g, u).contiguous()
                w.w_down = mat(up(H, 16), fp)
                put(w.w_down, 0, 0, get(p + "mlp.down", (H, f)))
            elif spec.mlp is not None:
                put(w.w_in, la.n_mix, 0, get(p + "mlp.up", (spec.mlp.ff, H)))
                put(w.w_o, 0, la.ff_col, get(p + "mlp.down", (H, spec.mlp.ff)))

    def weight_bytes(self) -> int:
        ts = [self.embed, self.bigram, self.embed_norm, self.lm_head, self.final_norm]
        for la in self.layers:
            for ns in [la.w] + [m.w for m in la.mixers]:
                ts += list(vars(ns).values())
        return sum(t.numel() * t.element_size() for t in ts if t is not None)

    # ------------------------------------------------------------------ what the engine sizes its caches by
    def cache_shapes(self) -> List[Optional[Tuple[int, int, int]]]:
        return [next((m.cache_shape() for m in la.mixers if m.cache_shape() is not None), None) for la in self.layers]

    def state_shapes(self):
        return [next((m.state_shape() for m in la.mixers if m.state_shape() is not None), None) for la in self.layers]

    def _mixers(self) -> List[Mixer]:
        return [m for la in self.layers for m in la.mixers]

    def decode_workspace(self, B: int, max_ctx: int, kv8=False) -> Dict[object, object]:
        """Split-K decode attention buffers per distinct head layout."""
        return workspaces(self._mixers(), B, max_ctx, self.device)

    def pass_items(self, lens: Sequence[int]):
        """Prefill-attention work lists of a pass's portions, per distinct kernel form."""
        return work_items(self._mixers(), lens, self.device)

    # ------------------------------------------------------------------ forward
    def _embed(self, b, kv) -> torch.Tensor:
        c = self.cfg
        if c.bigram is None:
            return ops.embed_pos(b.ids, b.positions, self.embed, c.embed_scale, self.pos_freq)
        return ops.embed_bigram(b.ids, b.segs, self.embed, self.bigram, c.embed_scale, c.bigram.mul_prev,
                                c.bigram.mul_cur, self.embed_norm, c.rms_eps, kv.state.last)

    def _mix(self, i: int, la: HybridLayer, x: torch.Tensor, b, kv) -> torch.Tensor:
        a = torch.empty(x.shape[0], la.k_out, dtype=self.dtype, device=self.device)
        if la.ff:
            u, gelu = ops.project_gelu(x, la.w.w_in, la.n_mix, a, la.ff_col, la.ff)
        else:
            gelu = None
            u = ops.project(x, la.w.w_in, "qkv")
            if la.ssm is None and la.k_mix < la.k_out:
                a[:, la.k_mix:].zero_()
        for m in la.mixers:
            if gelu is not None and m.takes_gelu:
                m.run(i, u, a, b, kv, self.cfg.rms_eps, gelu)
                gelu = None
            else:
                m.run(i, u, a, b, kv, self.cfg.rms_eps)
        if gelu is not None:
            ops.gelu_cols(u, gelu)
        return ops.project(a, la.w.w_o, "o")

    def _forward(self, b, kv) -> torch.Tensor:
        """All layers over the rows of batch ``b``; returns the final normed rows."""
        c = self.cfg
        b.rotary, b.shared = self.rotary, {}
        residual = self._embed(b, kv)
        src = None  # the last projection, not yet added to the residual
        for i, la in enumerate(self.layers):
            x = ops.add_norm32(residual, src, la.w.norm1, c.rms_eps, self.dtype, self.kp)
            if i and self.layer_hook is not None:
                self.layer_hook(i - 1, residual)
            src = self._mix(i, la, x, b, kv)
            if isinstance(la.spec.mlp, GLUSpec):
                m = la.spec.mlp
                x = ops.add_norm32(residual, src, la.w.norm2, c.rms_eps, self.dtype, self.kp)
                act = ops.project_glu(x, la.w.w_gu, m.limit, m.alpha, m.shift)
                src = ops.project(act, la.w.w_down, "down")
        x = ops.add_norm32(residual, src, self.final_norm, c.rms_eps, self.dtype, self.kp)
        if self.layer_hook is not None:
            self.layer_hook(len(self.layers) - 1, residual)
        return x

    def logits(self, x: torch.Tensor) -> torch.Tensor:
        return ops.logits32(x, self.lm_head)[:, :self.cfg.vocab_size]

    def forward_pass(self, x, kv, gather: bool = True, logits: bool = True) -> Optional[torch.Tensor]:
        """One packed batch (LLMEngine._pass_inputs): ``x.n_decode`` leading single tokens, then prompt portions.
        Logits of the rows ``x.last_rows``."""
        h = self._forward(x, kv)
        return self.logits(h.index_select(0, x.last_rows)) if logits else None

    def decode_pass(self, st, B: int, kv, workspace=None, gather: bool = True) -> torch.Tensor:
        """One token for each of the first ``B`` rows of the decode state ``st``."""
        segs = ops.Segments(st.state_slots[:B], st.positions[:B])
        b = SimpleNamespace(ids=st.next_ids[:B], positions=st.positions[:B], seq_idx=st.seq_idx[:B],
                            tables=st.block_tables[:B], decode_tables=st.block_tables[:B], n_decode=B,
                            workspace=workspace or {}, segs=segs)
        return self.logits(self._forward(b, kv))
