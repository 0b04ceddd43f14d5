"""The Muzozen design on the MI355X kernels against its float64 oracle (tests/muzozen_oracle.py): every mechanism alone,
then whole models in bf16 and fp32 through the engine's step function, scheduler and captured decode graphs."""
import math

import pytest
import torch

import muzozen_cases as M
import muzozen_oracle as O
from test_merulorn_gpu import BF, DEV, DTYPES, F32, dev, forms, rel, rnd, segments

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,buckets", [(64, 37), (51, 1), (4104, 1000)])
def test_bigram_embedding(dtype, width, buckets):
    """Portions, single rows and a sequence's first token; the pair of a portion's first token reaches back to the token
    that the slot remembers, whatever an earlier owner left there."""
    from llm_map_reduce_summarizer_amd import ops
    V = 40
    table, big, w = rnd(V, width, dtype=BF), rnd(buckets + 1, width, seed=1, dtype=BF), rnd(width, seed=2) + 1
    c = {"scale": 1.5, "bigram": {"buckets": buckets, "mul_prev": 1000003, "mul_cur": 17}}
    ids = torch.randint(0, V, (60,), generator=torch.Generator().manual_seed(4)).tolist()
    want = O.embed(ids, {"embed": table.double(), "bigram": big.double(), "embed.norm": w.double()}, c, 1e-4)
    last = torch.full((6,), 39, dtype=torch.int32, device=DEV)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)  # noqa: E731

    def run(at, end, seq):
        segs = seq if seq is not None else segments([end - at], [3], [at])
        return ops.embed_bigram(i32(ids[at:end]), segs, dev(table, dtype), dev(big, dtype), 1.5, 1000003, 17, dev(w), 1e-4,
                                last)
    cuts = [(0, 1), (1, 2), (2, 31), (31, 33), (33, 60)]
    got = [run(a, b, ops.Segments(i32([3]), i32([a])) if b == a + 1 else None) for a, b in cuts]
    assert float((torch.cat(got).double().cpu() - want).abs().max()) < 2e-5
    assert last.tolist() == [39, 39, 39, ids[-1], 39, 39]
    # several sequences in one batch
    segs = segments([1, 1, 40], [1, 2, 4], [0, 5, 0])
    last[2] = ids[9]
    out = ops.embed_bigram(i32([ids[0], ids[10]] + ids[:40]), segs, dev(table, dtype), dev(big, dtype), 1.5, 1000003, 17,
                           dev(w), 1e-4, last)
    ref = torch.cat([want[:1], want[10:11], want[:40]])
    assert float((out.double().cpu() - ref).abs().max()) < 2e-5
    assert last.tolist() == [39, ids[0], ids[10], ids[-1], ids[39], 39]


@pytest.mark.parametrize("N,F,K", [(128, 128, 128), (384, 1152, 256), (512, 3584, 512)])
def test_gelu_beside_the_projection(N, F, K):
    """Joint projection: plain columns and gelu columns, every row count's kernels, bf16 and 32-bit."""
    from llm_map_reduce_summarizer_amd import ops
    w = rnd(N + F, K, std=2 * K ** -0.5, dtype=BF)
    for T in (1, 5, 20, 40, 64, 65, 300):
        x = rnd(T, K, seed=T, dtype=BF)
        y = x.double() @ w.double().T
        want = O.gelu_tanh(y[:, N:])
        for dt in DTYPES:
            out = torch.full((T, 64 + F), 5.0, dtype=dt, device=DEV)
            u, job = ops.project_gelu(dev(x, dt), dev(w, dt), N, out, 64, F)
            if job is not None:
                ops.gelu_cols(u, job)
            rows = (u.double().sum(0) if u.dim() == 3 else u.double())[:, :N]
            assert rel(rows, y[:, :N]) < (4e-3 if dt == BF else 2e-6), (T, dt)
            assert rel(out[:, 64:], want) < (4e-3 if dt == BF else 2e-6), (T, dt)
            assert (out[:, :64] == 5).all()


def unrotate(x, pos, r):
    """The vector that ``rotate`` turns into ``x`` at ``pos``, up to the factor on cosine and sine squared."""
    freq, _ = O.rotation_frequencies(r)
    half, y = r["dims"] // 2, x.clone()
    for i in range(half):
        a = -pos * freq[i]
        u, v = x[..., i], x[..., i + half]
        y[..., i], y[..., i + half] = u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a)
    return y


# heads, dim, rot, vdim, kv_rank: flash and decode forms of every size, 32-bit only sizes, multiples of nothing
LATENT = [(8, 128, 64, 128, 512), (5, 40, 24, 56, 48), (3, 64, 64, 64, 128), (33, 32, 16, 40, 136), (2, 48, 16, 24, 256),
          (2, 136, 72, 200, 304), (3, 9, 6, 7, 11)]


@pytest.mark.parametrize("H,dim,rd,vdim,rank", LATENT)
@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_attention_finds_the_key_that_stands_out(H, dim, rd, vdim, rank, dtype):
    """Latent preparation and attention (expanded prompt portions, split-K decoded tokens, absorbed rows) over a paged
    cache whose unused rows hold large garbage: for chosen queries the first key, page-border keys, a far key or the
    query's own key carries the score, the rest of the weight is spread over hundreds of keys."""
    from llm_map_reduce_summarizer_amd import ops
    from llm_map_reduce_summarizer_amd.engine import mixers
    from llm_map_reduce_summarizer_amd.engine.config import LatentSpec, RotarySpec, YarnSpec
    from llm_map_reduce_summarizer_amd.ops.reference import rotary_table
    r = M.rot(rd, factor=3.0, original=100)
    s = r["scaling"]
    spec = LatentSpec(H, dim, vdim, 40, rank, RotarySpec(rd, r["base"], YarnSpec(s["factor"], s["original"], s["fast"],
                                                                                 s["slow"])), 0.7 * (dim + rd) ** -0.5)
    m = mixers.LatentMixer(spec, torch.device(DEV), dtype)
    cols = [0]

    def take(n):
        at = cols[0]
        cols[0] = -(-(at + n) // 8) * 8
        return at
    take(16)
    m.columns(take)
    ld = -(-cols[0] // 16) * 16
    wd = {"dq": rnd(40, 8, dtype=BF), "dq.norm": rnd(40, seed=1) + 1, "dkv": rnd(rank + rd, 8, dtype=BF),
          "dkv.norm": rnd(rank, seed=2, std=0.2) + 1, "uq": rnd(H * (dim + rd), 40, seed=3, dtype=BF),
          "uk": rnd(H * dim, rank, seed=4, std=rank ** -0.5, dtype=BF),
          "uv": rnd(H * vdim, rank, seed=5, std=rank ** -0.5, dtype=BF), "o": rnd(8, H * vdim, dtype=BF)}
    loader = mixers.Loader(lambda n, shape: wd[n].view(shape), torch.device(DEV), dtype)
    w_in, w_o = loader.mat(ld, 8), loader.mat(16, m.width)
    m.load(loader, "", w_in, w_o, 8)
    cs = rotary_table(2000, spec.rot, DEV)
    lens = [300, 97, 64, 65, 1]
    page, npg, ncol = 64, 40, -(-H * m.qw // 16) * 16
    tables = torch.zeros(len(lens), 8, dtype=torch.int32)
    perm, at = (torch.randperm(npg - 1, generator=torch.Generator().manual_seed(1)) + 1).tolist(), 0
    us, qs, c = [], [], {"heads": H, "dim": dim, "vdim": vdim, "rot": r, "scale": spec.scale}
    wk, wv = wd["uk"].double(), wd["uv"].double()
    for i, n in enumerate(lens):
        need = -(-n // page)
        tables[i, :need] = torch.tensor(perm[at: at + need], dtype=torch.int32)
        at += need
        u = rnd(n, ld, seed=10 + i).to(BF).double()
        u[:, m.dkv + rank: m.dkr] = 0  # columns that pad a section are zero in a projection
        lat, kr = latents_of(u, m, wd, rank, rd, r)
        q = rnd(n, H, dim + rd, seed=20 + i).double()
        for t, j in ((n - 1, 0), (n - 1 - n // 3, 63), (n // 2, n // 2), (n - 2, 64), (n // 3, 1)):
            if 0 <= j <= t < n:
                q[t, :, :dim] = 4.0 * (lat[j] @ wk.T).view(H, dim)
                q[t, :, dim:] = 4.0 * unrotate(kr[j], t, r)
        us.append(u)
        qs.append(q)
    T = sum(lens)
    qrow = torch.zeros(T, ncol, dtype=torch.float64)
    qv = qrow[:, :H * m.qw].view(T, H, m.qw)
    qv[:, :, :dim], qv[:, :, m.dim8: m.dim8 + rd] = torch.cat(qs)[:, :, :dim], torch.cat(qs)[:, :, dim:]
    pos = torch.cat([torch.arange(n) for n in lens]).int().to(DEV)
    seq = torch.cat([torch.full((n,), i) for i, n in enumerate(lens)]).int().to(DEV)
    bt = tables.to(DEV)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)  # noqa: E731
    tol = 1.5e-2 if dtype == BF else 2e-5
    for (usrc, dt, uvals), (qsrc, _, qvals) in zip(forms(torch.cat(us).float()), forms(qrow.float())):
        if dt != dtype:
            continue
        cache = torch.full((npg, 1, page, m.row), 40.0, dtype=dtype, device=DEV)
        cq = ops.latent_prep(usrc, m, m.w.dq_norm, m.w.dkv_norm, 1e-5, cs, pos, seq, bt, cache, page, dtype)
        assert rel(cq[:, :40], O.rms_norm(uvals[:, m.dq: m.dq + 40], wd["dq.norm"].double(), 1e-5)) < \
            (4e-3 if dtype == BF else 1e-6) and not cq[:, 40:].any()
        want, b = [], 0
        for i, n in enumerate(lens):
            lat, kr = latents_of(uvals[b: b + n], m, wd, rank, rd, r)
            row = cache[bt[i].long(), 0].reshape(-1, m.row)[:n]
            assert rel(row[:, :rank], lat) < (4e-3 if dtype == BF else 1e-6)
            assert rel(row[:, m.rank8: m.rank8 + rd], kr) < (4e-3 if dtype == BF else 2e-6)
            qq = qvals[b: b + n, :H * m.qw].view(n, H, m.qw)
            qq = torch.cat([qq[:, :, :dim], qq[:, :, m.dim8: m.dim8 + rd]], -1)
            want.append(O.latent_attend(qq, lat, kr, wk, wv, c))
            b += n
        want = torch.cat(want)

        def same(out, rows, what):
            assert (out[:, :8] == 7).all() and (out[:, 8 + H * m.vp:] == 7).all(), what
            o = out[:, 8: 8 + H * m.vp].reshape(-1, H, m.vp)[:, :, :vdim].reshape(len(rows), -1)
            for k, t in enumerate(rows):
                assert rel(o[k], want[t]) < tol, (what, t)

        def blank(n):
            return torch.full((n, H * m.vp + 16), 7.0, dtype=dtype, device=DEV)
        qa = ops.latent_absorb(qsrc, T, m, m.w.w_uk, cs, pos, dtype)
        out = blank(T)
        ops.latent_out(ops.latent_rows(qa, cache, pos, seq, bt, H, m.rank8, page, spec.scale), m, m.w.w_uv, out, 8)
        same(out, list(range(T)), "absorbed rows")
        last = [sum(lens[:i + 1]) - 1 for i in range(len(lens))]
        if m.mfma:
            ix = torch.tensor(last, device=DEV)
            for splits in (1, 2, 3, 7):
                ws = ops.latent_workspace(len(last), H, m.rank8, 512, DEV)
                ws.splits = splits
                ws.part_o = torch.full((len(last) * H * splits * m.rank8,), float("nan"), device=DEV)
                ws.part_ml = torch.full((len(last) * H * splits * 2,), float("nan"), device=DEV)
                parts = ops.latent_decode(qa[ix].contiguous(), cache, bt, pos[ix].contiguous(), H, m.rank8, page,
                                          spec.scale, ws)
                out = blank(len(last))
                ops.latent_out_parts(parts, m, m.w.w_uv, out, 8)
                same(out, last, "decode %d" % splits)
            many = ix.repeat(26)  # enough rows that a merging block takes several
            parts = ops.latent_decode(qa[many].contiguous(), cache, bt.repeat(26, 1), pos[many].contiguous(), H, m.rank8, page,
                                      spec.scale, None)
            out = blank(len(many))
            ops.latent_out_parts(parts, m, m.w.w_uv, out, 8)
            same(out, last * 26, "decode of many rows")
        if not m.flash or (qsrc.dim() == 3 and T > 64 and H > 8):
            continue
        for nd in ((0, 3) if H < 9 else (0,)):
            for pre in ([0] * len(lens), [101, 64, 62, 1, 0]):
                part = [n - p for n, p in zip(lens, pre)]
                rows = [sum(lens[:i]) + p + k for i, (n, p) in enumerate(zip(lens, pre)) for k in range(n - p)]
                ix = torch.tensor(list(range(nd)) + rows, device=DEV)
                qsub = (qsrc[:, ix] if qsrc.dim() == 3 else qsrc[ix]).contiguous()
                ctx = ops.PortionContext(part, pre, list(range(len(lens))), torch.device(DEV))
                lat = ops.latent_gather(cache, ctx, bt, m.lat, page)
                qr = ops.latent_rope(qsub, nd, m, cs, pos[ix].contiguous())
                out = blank(len(rows))
                ops.latent_prefill(qr, ops.latent_expand(lat, m.w.w_kv), lat, ctx, m,
                                   i32([0] + torch.tensor(part).cumsum(0).tolist()), part,
                                   ops.latent_items(part, ops.latent_block_rows(m.qw, m.vp)).to(DEV), spec.scale, out, 8)
                same(out, rows, "portion")


def latents_of(u, m, wd, rank, rd, r):
    """The oracle's latents fed with given projection columns: an identity stands where the weights would be."""
    x = torch.cat([u[:, m.dkv: m.dkv + rank], u[:, m.dkr: m.dkr + rd]], 1)
    w = {"dkv": torch.eye(rank + rd, dtype=torch.float64), "dkv.norm": wd["dkv.norm"].double()}
    return O.latents(x, w, "", {"kv_rank": rank, "rot": r}, 1e-5)


def test_latent_kernels_of_real_sizes_are_the_fused_ones():
    from llm_map_reduce_summarizer_amd.ops import hip
    assert hip.latent_prefill_form(192, 128) == (12, 256) and hip.latent_decode_form(512, 576) is not None
    assert hip.latent_prefill_form(208, 128) is None and hip.delta_chunk_ok(128, 128)


# heads, key heads, dim, vdim
DELTA = [(4, 2, 128, 128), (3, 3, 24, 40), (2, 1, 64, 136), (6, 2, 32, 16), (2, 2, 200, 112), (3, 1, 5, 7), (2, 1, 256, 64)]


@pytest.mark.parametrize("H,G,dim,vdim", DELTA)
@pytest.mark.parametrize("dtype", DTYPES)
def test_delta_rule(H, G, dim, vdim, dtype, monkeypatch):
    """Decoded rows, short and long portions, fresh and continued slots holding garbage or carried state, keys that repeat
    (so that corrections chain through a chunk), decays from almost none to total, output norm and gate."""
    from llm_map_reduce_summarizer_amd import ops
    from llm_map_reduce_summarizer_amd.engine import mixers
    from llm_map_reduce_summarizer_amd.engine.config import DeltaSpec
    from llm_map_reduce_summarizer_amd.ops import hip
    m = mixers.DeltaMixer(DeltaSpec(H, G, dim, vdim, 2), torch.device(DEV), dtype)
    cols = [0]

    def take(n):
        at = cols[0]
        cols[0] = -(-(at + n) // 8) * 8
        return at
    m.columns(take)
    m.col = 16
    ld = -(-cols[0] // 16) * 16
    lens = [1, 1, 2, 65, 200, 64]
    T = sum(lens)
    x = rnd(T, m.channels, std=0.8)
    k = x[:, m.xk: m.xk + G * dim]
    k[50:80] = k[50] + 0.05 * k[50:80]  # nearly one direction
    k[100:110] = 0.0
    x = x.to(dtype)
    u = rnd(T, ld, seed=1, std=1.5)
    u[60:70, m.b: m.b + H] = 9.0  # step size almost one
    dt_bias, A_log, norm = rnd(H, seed=2, std=1.5) - 3, rnd(H, seed=3, std=1.5), rnd(vdim, seed=4, std=0.2) + 1
    A_log[0], u[90, m.a] = 4.0, 30.0  # a decay that forgets everything
    slots, pos0 = [3, 1, 5, 2, 6, 4], [9, 0, 7, 64, 0, 1000]
    init = rnd(len(lens), H, dim, vdim, seed=6, std=0.5)
    N4 = dim + (-dim) % 4
    sets = [s for s in forms(u) if s[1] == dtype]
    if dtype == BF and hip.delta_chunk_ok(vdim, dim):  # every form of the chunked kernel
        waves = [(8, 0), (4, 0), (4, 1), (2, 0), (2, 1)] if dim <= 128 else [(4, 0), (2, 0)]
        sets = [s + (w,) for s, w in zip(sets * len(waves), waves + waves[::-1])]
    for src, dt_, vals, *w in sets:
        if w:
            monkeypatch.setattr(hip, "delta_waves", lambda *_, w=w[0]: w)
        state = torch.full((8, H, vdim, N4), 1e4, device=DEV)
        state[..., dim:] = 0
        for i, s in enumerate(slots):
            if pos0[i]:
                state[s, ..., :dim] = init[i].transpose(1, 2).to(DEV)
        a = torch.full((T, m.col + m.width + 8), 7.0, dtype=dtype, device=DEV)
        ops.delta_mix(dev(x), src, m, dev(-torch.exp(A_log)), dev(dt_bias), dev(norm), 1e-3, state,
                      segments(lens, slots, pos0), a)
        assert (a[:, :m.col] == 7).all() and (a[:, m.col + m.width:] == 7).all()
        assert not a[:, m.col + H * vdim: m.col + m.width].any()
        f, b = x.double(), 0
        for i, n in enumerate(lens):
            e = b + n
            q = O.unit(f[b:e, :G * dim].view(n, G, dim)) * dim ** -0.5
            kk = O.unit(f[b:e, m.xk: m.xk + G * dim].view(n, G, dim))
            v = f[b:e, m.xv: m.xv + H * vdim].view(n, H, vdim)
            ldec = -torch.exp(A_log.double()) * O.softplus(vals[b:e, m.a: m.a + H] + dt_bias.double())
            o, S = O.delta_rule(q, kk, v, O.logistic(vals[b:e, m.b: m.b + H]), ldec,
                                init[i].double() if pos0[i] else None)
            want = O.head_norm_gate(o, vals[b:e, m.g: m.g + H * vdim].view(n, H, vdim), norm.double(), 1e-3)
            got = a[b:e, m.col: m.col + H * vdim]
            assert rel(got, want.reshape(n, -1)) < (4e-3 if dtype == BF else 1e-5), ("out", i)
            tol = 1e-4 if dtype == BF else 1e-5
            assert rel(state[slots[i], ..., :dim], S.transpose(1, 2)) < tol, ("state", i)
            b = e


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("name", sorted(M.CONFIGS))
@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_and_token_by_token(name, dtype, tmp_path):
    eng = M.engine(name, tmp_path, DEV, dtype)
    ids = M.tokens(name, 140)
    want = M.expected(name, ids)
    M.check(M.feed(eng, "a", ids, [140]), want, dtype, "one portion")
    M.check(M.feed(eng, "b", ids, [1] * 140), want, dtype, "token by token")
    M.check(M.feed(eng, "c", ids, M.cuts(140, [2, 3, 64, 1, 17])), want, dtype, "portions")


@pytest.mark.parametrize("name", ["mixed", "wide"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_requests_share_batches_and_reuse_slots(name, dtype, tmp_path):
    lengths = {"a": 131, "b": 5, "c": 64, "d": 1, "e": 90, "f": 65}
    eng = M.engine(name, tmp_path, DEV, dtype, max_num_seqs=3, kv_pages=8)
    reqs = {r: M.tokens(name, n, seed=i) for i, (r, n) in enumerate(lengths.items())}
    got = M.feed_mixed(eng, reqs, M.mixed_plan(lengths, [1, 30, 2, 1, 64, 1], live=3))
    for r, ids in reqs.items():
        M.check(got[r], M.expected(name, ids), dtype, r)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompt_then_long_decoding(dtype, tmp_path):
    """A prompt of several query blocks and many chunks, then 100 decoded tokens across page borders."""
    eng = M.engine("wide", tmp_path, DEV, dtype, max_model_len=1024)
    ids = M.tokens("wide", 700)
    M.check(M.feed(eng, "a", ids, [600] + [1] * 100), M.expected("wide", ids), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_of_more_than_a_thousand_rows(dtype, tmp_path):
    """Row counts from which on the preparation and norm kernels change their form, in one portion and in three."""
    eng = M.engine("mixed", tmp_path, DEV, dtype, max_model_len=1280)
    ids = M.tokens("mixed", 1130)
    want = M.expected("mixed", ids)
    M.check(M.feed(eng, "a", ids, [1100] + [1] * 30), want, dtype, "one portion")
    M.check(M.feed(eng, "b", ids, [70, 1030, 2] + [1] * 28), want, dtype, "portions")


@pytest.mark.parametrize("name", ["mixed", "wide"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_with_graphs(name, dtype, tmp_path):
    """generate(): packed prefill, hipGraph decode replayed over growing, shrinking and refilled batches (several
    captures, eager work between replays), sliced prompts, requests joining a running batch."""
    from llm_map_reduce_summarizer_amd.engine.engine import SamplingParams
    eng = M.engine(name, tmp_path, DEV, dtype, prefill_chunk=64, max_num_seqs=3)
    prompts = [M.tokens(name, n, seed=n) for n in (3, 130, 64, 1, 77)]
    slack = 0.15 if dtype == BF else 1e-4
    for _ in range(2):
        outs = eng.generate(prompts, [SamplingParams(n, 0.0, 1) for n in (30, 12, 6, 20, 2)])
        assert [len(o.token_ids) for o in outs] == [30, 12, 6, 20, 2]
        for p, o in zip(prompts, outs):
            M.check_greedy(name, p, o.token_ids, slack)
    fed = []

    def feeder(done):
        if not fed:
            fed.append(1)
            return [(p, SamplingParams(7, 0.0, 1)) for p in prompts[1:3]]
        return []
    outs = eng.generate(prompts[:1], [SamplingParams(25, 0.0, 1)], feeder=feeder)
    for p, o in zip([prompts[0]] + prompts[1:3], outs):
        M.check_greedy(name, p, o.token_ids, slack)
    assert eng.stats["graph_captures"] >= 2 and eng.kv.state.alloc.available() == 3


def test_graph_capture_leaves_live_state_alone(tmp_path):
    """The eager warm-up before a capture must not advance the state (last tokens included) of the rows it runs on."""
    from llm_map_reduce_summarizer_amd.engine.engine import SamplingParams
    prompts = [M.tokens("wide", n, seed=n) for n in (50, 20)]
    outs = []
    for graphs in (False, True):
        eng = M.engine("wide", tmp_path, DEV, F32, use_graphs=graphs)
        outs.append([o.token_ids for o in eng.generate(prompts, [SamplingParams(40, 0.0, 1)] * 2)])
    assert outs[0] == outs[1]
