"""Plain float64 implementation of the Muzozen design, one function per mechanism, token by token where the
mechanism is a recurrence.  It is what the engine is compared with and shares no code with it: tensors come from
a dict of named arrays, every loop is written out, and nothing is fused, absorbed, cached, paged or batched.

``planted`` (a set of names) switches on deliberate mistakes, so that tests can show that their inputs would
reveal them."""
import math

import torch

F = torch.float64


def logistic(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def silu(z):
    return z * logistic(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x, weight, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def bigram_row(prev, cur, c):
    """Row of the bigram table for the pair (prev, cur); the row after the last bucket for a first token."""
    return c["buckets"] if prev is None else (prev * c["mul_prev"] + cur * c["mul_cur"]) % c["buckets"]


def embed(ids, w, c, eps, planted=()):
    rows = []
    for t, tok in enumerate(ids):
        prev = ids[t - 1] if t else None
        if "first_pair_zero" in planted and t == 0:
            prev = 0
        rows.append(w["embed"][tok] * c["scale"] + w["bigram"][bigram_row(prev, tok, c["bigram"])])
    return rms_norm(torch.stack(rows), w["embed.norm"], eps)


def rotation_frequencies(rot):
    """Angular frequencies of the rotated pairs and the factor on cosine and sine (YaRN interpolation)."""
    dims, base, s = rot["dims"], rot["base"], rot.get("scaling")
    out = []
    if s is not None:
        def dim_of(turns):
            return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
        lo = max(math.floor(dim_of(s["fast"])), 0)
        hi = min(math.ceil(dim_of(s["slow"])), dims - 1)
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if s is not None:
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / s["factor"] * ramp + f * (1.0 - ramp)
        out.append(f)
    return out, (1.0 if s is None else 0.1 * math.log(s["factor"]) + 1.0)


def rotate(x, pos, rot, planted=()):
    """Rotate-half pairs (i, i + dims / 2) of the vector x at position ``pos``."""
    freq, m = rotation_frequencies(rot)
    if "plain_rotation" in planted:
        freq, m = rotation_frequencies({"dims": rot["dims"], "base": rot["base"]})
    half = rot["dims"] // 2
    y = x.clone()
    for i in range(half):
        a = pos * freq[i]
        u, v = x[..., i], x[..., i + half]
        y[..., i] = m * (u * math.cos(a) - v * math.sin(a))
        y[..., i + half] = m * (v * math.cos(a) + u * math.sin(a))
    return y


def latents(h, w, pre, c, eps, planted=()):
    """(normed latents [T, kv_rank], rotated shared key part [T, rot_dim]) of a layer that has its own."""
    kv = h @ w[pre + "dkv"].T
    r = c["kv_rank"]
    lat = rms_norm(kv[:, :r], w[pre + "dkv.norm"], eps)
    return lat, torch.stack([rotate(kv[t, r:], t, c["rot"], planted) for t in range(h.shape[0])])


def latent_queries(h, w, pre, c, eps):
    cq = rms_norm(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps)
    return (cq @ w[pre + "uq"].T).view(h.shape[0], c["heads"], c["dim"] + c["rot_dim"])


def latent_attend(q, lat, kr, w_uk, w_uv, c, planted=()):
    """Causal softmax attention of raw queries [T, heads, dim + rot_dim] over latents and rotated key parts, one
    head after the other.  Returns [T, heads * vdim]."""
    T, H, d, dv = q.shape[0], c["heads"], c["dim"], c["vdim"]
    out = torch.zeros(T, H * dv, dtype=F)
    qr = torch.stack([rotate(q[i, :, d:], i, c["rot"], planted) for i in range(T)])
    for a in range(H):
        k = lat @ w_uk[a * d:(a + 1) * d].T
        v = lat @ w_uv[a * dv:(a + 1) * dv].T
        for i in range(T):
            s = (k[:i + 1] @ q[i, a, :d] + kr[:i + 1] @ qr[i, a]) * c["scale"]
            if "drop_first_key" in planted and i > 0:
                s[0] = -math.inf
            p = torch.exp(s - s.max())
            out[i, a * dv:(a + 1) * dv] = (p / p.sum()) @ v[:i + 1]
    return out


def latent_attention(h, w, pre, c, eps, shared, planted=()):
    """``shared``: what another layer's ``latents`` returned, or None for a layer with its own.  Returns (output,
    the latents it used)."""
    own = latents(h, w, pre, c, eps, planted) if shared is None else shared
    q = latent_queries(h, w, pre, c, eps)
    o = latent_attend(q, own[0], own[1], w[pre + "uk"], w[pre + "uv"], c, planted)
    return o @ w[pre + "o"].T, own


def short_conv(u, kernel):
    """Per-channel causal convolution; the last tap multiplies the current token, zeros stand before the start."""
    T, taps = u.shape[0], kernel.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += kernel[:, j] * u[s]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, log_decay, S=None, planted=()):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, head after head.  q, k [T, kv heads, dim] (as they
    enter the recurrence), v [T, heads, vdim], beta and log_decay [T, heads]; S [heads, dim, vdim] or None (zero).
    Returns (o [T, heads, vdim], S after the last token)."""
    T, H = beta.shape
    rep = H // k.shape[1]
    S = torch.zeros(H, k.shape[2], v.shape[2], dtype=F) if S is None else S.clone()
    o = torch.zeros(T, H, v.shape[2], dtype=F)
    for a in range(H):
        g = a // rep
        s = S[a]
        for t in range(T):
            if "state_reset_64" in planted and t % 64 == 0:
                s = torch.zeros_like(s)
            s = torch.exp(log_decay[t, a]) * s
            if "read_before_write" in planted:
                o[t, a] = s.T @ q[t, g]
            u = beta[t, a] * (v[t, a] - s.T @ k[t, g])
            s = s + torch.outer(k[t, g], u)
            if "read_before_write" not in planted:
                o[t, a] = s.T @ q[t, g]
        S[a] = s
    return o, S


def delta_inputs(h, w, pre, c):
    """What enters the recurrence: unit queries (times dim^-1/2) and keys, values, step sizes, log decays."""
    T, H, G, d, dv = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(short_conv(h @ w[pre + n].T, w[pre + n + ".conv"])) for n in "qkv")
    q = unit(q.view(T, G, d)) * d ** -0.5
    k = unit(k.view(T, G, d))
    beta = logistic(h @ w[pre + "b"].T)
    ld = -torch.exp(w[pre + "A_log"]) * softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"])
    return q, k, v.view(T, H, dv), beta, ld


def head_norm_gate(o, gate, weight, eps):
    """Each head's output over its root mean square, times the shared weight, times silu(gate)."""
    return rms_norm(o, weight, eps) * silu(gate)


def delta_mixer(h, w, pre, c, eps, planted=()):
    T, H, dv = h.shape[0], c["heads"], c["vdim"]
    o, _ = delta_rule(*delta_inputs(h, w, pre, c), planted=planted)
    gate = (h @ w[pre + "g"].T).view(T, H, dv)
    return head_norm_gate(o, gate, w[pre + "norm"], eps).reshape(T, H * dv) @ w[pre + "o"].T


def feed_forward(h, w, pre):
    return gelu_tanh(h @ w[pre + "up"].T) @ w[pre + "down"].T


def forward(cfg, weights, ids, planted=(), layers_out=None):
    """Logits [T, vocab] (float64) of one sequence from its start; ``layers_out`` collects the residual stream
    after every layer."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = embed(ids, w, cfg["embedding"], eps, planted)
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % i
        h = rms_norm(x, w[p + "norm1"], eps)
        m = layer["mixer"]
        if layer["type"] == "delta":
            y = delta_mixer(h, w, p + "mix.", m, eps, planted)
        else:
            y, kept[i] = latent_attention(h, w, p + "mix.", m, eps, kept[m["kv_from"]] if "kv_from" in m else None,
                                          planted)
        if layer["mlp"] is not None:
            y = y + feed_forward(h, w, p + "mlp.")
        x = x + y
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
