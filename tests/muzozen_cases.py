"""Small Muzozen configurations, random weights and schedules shared by the CPU and GPU tests of the design."""
import functools
import json
import os

import torch

import muzozen_oracle as O
from merulorn_cases import TOL, check, cuts, error, feed, feed_mixed, mixed_plan  # noqa: F401


def rot(dims, base=10000.0, factor=4.0, original=64, fast=8.0, slow=0.5):
    return {"dims": dims, "base": base,
            "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow} if factor else None}


def latent(heads, dim, vdim, q_rank, kv_rank, r, scale=None, kv_from=None, ff=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot_dim": r["dims"], "rot": r,
         "scale": scale or 1.2 * (dim + r["dims"]) ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": dense(ff)}


def delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return {"type": "delta", "mlp": dense(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def config(vocab, width, layers, buckets, muls=(37, 11), eps=1e-5, scale=0.7):
    return {"architecture": "Muzozen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
            "embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": muls[0], "mul_cur": muls[1]}}}


CONFIGS = {
    # shared latents across other layers, head sizes that differ between the sharing layers, with and without feed-forward
    "mixed": config(301, 144, [
        latent(6, 40, 56, 72, 48, rot(24), ff=104),
        delta(4, 2, 24, 40, 4, ff=72),
        latent(4, 32, 24, 40, 48, rot(24), scale=0.3, kv_from=0),
        latent(3, 48, 64, 96, 88, rot(8, base=500.0, factor=2.0, original=32), ff=136),
        delta(6, 3, 40, 16, 2),
        latent(2, 16, 32, 24, 48, rot(24), kv_from=0, ff=40),
        latent(5, 24, 40, 56, 88, rot(8, base=500.0, factor=2.0, original=32), kv_from=3)], buckets=211),
    # sizes that are multiples of nothing; one convolution tap; one head per key head; plain rotation
    "odd": config(77, 50, [
        delta(3, 3, 5, 7, 1, ff=36),
        latent(3, 9, 7, 13, 11, rot(6, factor=None), ff=20),
        latent(1, 6, 5, 7, 11, rot(6, factor=None), kv_from=1),
        delta(2, 1, 9, 3, 5)], buckets=1, muls=(1, 1), eps=1e-3, scale=1.0),
    # head sizes of real models
    "wide": config(130, 256, [
        latent(8, 128, 128, 192, 512, rot(64, base=500000.0), ff=192),
        delta(4, 2, 128, 128, 4, ff=256),
        latent(8, 128, 128, 192, 512, rot(64, base=500000.0), kv_from=0)], buckets=503),
    # more heads than a decode workgroup takes; medium latents; wide delta values
    "many_heads": config(65, 96, [
        latent(40, 64, 48, 64, 200, rot(32), ff=64),
        delta(2, 1, 64, 136, 3, ff=64),
        latent(2, 40, 16, 24, 200, rot(32), kv_from=0)], buckets=97),
    # heads and latents wider than the flash kernel takes, wide delta keys
    "huge_heads": config(65, 96, [
        latent(2, 136, 200, 72, 304, rot(72)),
        delta(3, 3, 200, 112, 2, ff=48)], buckets=53),
}


@functools.lru_cache(maxsize=None)
def weights(name, seed=0):
    """Random weights loud enough that every mechanism moves the logits: sharp attention, step sizes and decays over
    their whole range, a bigram table as loud as the embedding."""
    cfg = CONFIGS[name]
    g = torch.Generator().manual_seed(2000 + seed)
    W = cfg["width"]

    def rn(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)
    b = cfg["embedding"]["bigram"]["buckets"]
    w = {"embed": rn(cfg["vocab"], W), "bigram": rn(b + 1, W, std=0.7), "embed.norm": rn(W, std=0.2, mean=1.0),
         "head": rn(cfg["vocab"], W, std=W ** -0.5), "final.norm": rn(W, std=0.2, mean=1.0)}
    for i, la in enumerate(cfg["layers"]):
        p, m = "l%d." % i, la["mixer"]
        x = p + "mix."
        w[p + "norm1"] = rn(W, std=0.2, mean=1.0)
        if la["type"] == "delta":
            kd, vd = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, rows in (("q", kd), ("k", kd), ("v", vd)):
                w[x + n] = rn(rows, W, std=W ** -0.5)
                w[x + n + ".conv"] = rn(rows, m["conv"], std=0.7)
            for n, rows in (("b", m["heads"]), ("a", m["heads"]), ("g", vd)):
                w[x + n] = rn(rows, W, std=1.5 * W ** -0.5)
            w[x + "A_log"] = rn(m["heads"], std=1.0)
            w[x + "dt_bias"] = rn(m["heads"], std=1.0, mean=-3.0)
            w[x + "norm"] = rn(m["vdim"], std=0.2, mean=1.0)
            w[x + "o"] = rn(W, vd, std=1.5 * vd ** -0.5)
        else:
            H, r = m["heads"], m["rot_dim"]
            w[x + "dq"] = rn(m["q_rank"], W, std=W ** -0.5)
            w[x + "dq.norm"] = rn(m["q_rank"], std=0.2, mean=1.1)
            w[x + "uq"] = rn(H * (m["dim"] + r), m["q_rank"], std=m["q_rank"] ** -0.5)
            if "kv_from" not in m:
                w[x + "dkv"] = rn(m["kv_rank"] + r, W, std=W ** -0.5)
                w[x + "dkv.norm"] = rn(m["kv_rank"], std=0.2, mean=1.0)
            w[x + "uk"] = rn(H * m["dim"], m["kv_rank"], std=m["kv_rank"] ** -0.5)
            w[x + "uv"] = rn(H * m["vdim"], m["kv_rank"], std=m["kv_rank"] ** -0.5)
            w[x + "o"] = rn(W, H * m["vdim"], std=1.5 * (H * m["vdim"]) ** -0.5)
        if la["mlp"] is not None:
            ff = la["mlp"]["ff"]
            w[p + "mlp.up"] = rn(ff, W, std=1.3 * W ** -0.5)
            w[p + "mlp.down"] = rn(W, ff, std=ff ** -0.5)
    return w


def tokens(name, n, seed=0):
    g = torch.Generator().manual_seed(8000 + seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


_EXPECTED = {}


def expected(name, ids, planted=()):
    """The oracle's logits [T, vocab] (cached per prompt)."""
    key = (name, tuple(ids), tuple(planted))
    if key not in _EXPECTED:
        _EXPECTED[key] = O.forward(CONFIGS[name], weights(name), list(ids), planted)
    return _EXPECTED[key]


def checkpoint(name, folder):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    save_file({k: v.contiguous() for k, v in weights(name).items()}, os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(CONFIGS[name], f)
    return str(folder)


def engine(name, folder, device, dtype, **kw):
    from llm_map_reduce_summarizer_amd.engine.engine import LLMEngine
    from llm_map_reduce_summarizer_amd.engine.registry import load_config
    path = checkpoint(name, folder)
    opts = dict(max_num_seqs=4, max_model_len=512, kv_pages=33, eos_ids=(), sync_every=4, max_new_cap=256)
    opts.update(kw)
    return LLMEngine(load_config(path), device=device, dtype=dtype, weights_path=path, **opts)


def check_greedy(name, prompt, out, slack):
    """Every generated token is the oracle's best next token given the ones before it, up to ``slack`` (in units of
    the logits' root mean square)."""
    lg = expected(name, list(prompt) + list(out))
    rms = lg.pow(2).mean().sqrt()
    for k, tok in enumerate(out):
        row = lg[len(prompt) - 1 + k]
        gap = float((row.max() - row[tok]) / rms)
        assert gap <= slack, "token %d of %d: %.3g below the best" % (k, len(out), gap)
