"""Every mechanism of the Pifutar design alone: the package's torch operations (CPU) and its HIP kernels (`gpu` marker)
against the plain float64 functions of `pifutar_oracle`, on small inputs made here."""
import pytest
import torch

import pifutar_oracle as O

F64 = torch.float64


def rnd(*shape, seed=0, std=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64) * std


def close(got, ref, tol=2e-5):
    ref = ref.to(F64)
    err = (got.detach().cpu().to(F64) - ref).abs().max().item() / max(1.0, ref.abs().max().item())
    assert err < tol, err


# ---- torch operations (the CPU executor's) ---------------------------------------------------------------------------
def test_linear_attention_in_portions():
    from distributed_llm_inference_amd.ops import reference as R
    T, H, d, dv = 50, 3, 6, 10
    q, k, v, ld = rnd(T, H, d, seed=1), rnd(T, H, d, seed=2), rnd(T, H, dv, seed=3), -rnd(T, H, d, seed=4).exp()
    ref, S, outs, t0 = O.linear_attention(q, k, v, ld), torch.zeros(H, d, dv), [], 0
    for c in (1, 2, 17, 1, 29):
        sl = slice(t0, t0 + c)
        o, S = R.linear_attention(q[sl].float(), k[sl].float(), v[sl].float(), ld[sl].float(), S)
        outs.append(o)
        t0 += c
    close(torch.cat(outs), ref)


@pytest.mark.parametrize("taps", [1, 2, 3, 6])
def test_input_convolution_in_portions(taps):
    from distributed_llm_inference_amd.ops import reference as R
    T, H = 20, 12
    h, w = rnd(T, H, seed=1), rnd(H, taps, seed=2)
    ref, prev, outs, t0 = O.input_conv(h, w), torch.zeros(taps - 1, H), [], 0
    for c in (1, 1, 2, 5, 1, 10):
        x = h[t0:t0 + c].float()
        y, prev = R.short_conv(x, prev, w.float())
        outs.append(x + y)
        t0 += c
    close(torch.cat(outs), ref)


def test_polynomial_of_normed_powers():
    from distributed_llm_inference_amd.ops import reference as R
    z, c = rnd(9, 40, seed=1, std=2.0), torch.tensor([0.5, -0.3, 0.7, 0.2], dtype=F64)
    close(R.poly_norm(z.float(), c.float(), 1e-5), O.poly_norm(z, 1e-5, c))


def test_rotation_of_neighbouring_pairs_and_window():
    from distributed_llm_inference_amd.models.rope import rope_table
    from distributed_llm_inference_amd.ops import reference as R
    x, pos = rnd(6, 2, 14, seed=6), torch.tensor([0, 1, 2, 50, 700, 703])
    for dims, base in ((14, 100.0), (6, 500000.0)):
        cos, sin = rope_table(dims, base, None, 710)
        close(R.rope_partial(x.float(), cos, sin, pos, True), O.rotate_pairs(x, pos, dims, base), 1e-5)
    q, k, v = rnd(60, 2, 8, seed=7), rnd(60, 2, 8, seed=8), rnd(60, 2, 5, seed=9)
    for win in (1, 7, 32, 33, 0):
        s = (torch.einsum("ihd,jhd->hij", q, k) * 0.3).masked_fill(~O.window_mask(60, win), float("-inf"))
        close(R.attention(q.float(), k.float(), v.float(), 0, 0.3, window=win), torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v))


# ---- HIP kernels ------------------------------------------------------------------------------------------------------
def _K():
    from distributed_llm_inference_amd import ops
    return ops.load()


def _meta(seqs, dev="cuda"):
    """seqs: [(slot, q_len, ctx)] -> tok_pos, tok_seq, q_start, ctx, slots (int32 on the device)."""
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
    qs = [0]
    for _, n, _ in seqs:
        qs.append(qs[-1] + n)
    return (i32([c + i for _, n, c in seqs for i in range(n)]), i32([s for s, n, _ in seqs for _ in range(n)]), i32(qs),
            i32([c for _, _, c in seqs]), i32([s for s, _, _ in seqs]))


# requests (slot, length) in steps of (request, tokens): portions of two tokens, single tokens beside portions, steps of single
# tokens alone, portions shorter and longer than any ring, a slot taken over by another request
REQS = {"a": (2, 90), "b": (0, 75), "c": (2, 40)}
STEPS = [[("a", 1)], [("a", 2), ("b", 3)], [("a", 1), ("b", 1)], [("a", 1), ("b", 1)], [("b", 2), ("a", 66)], [("a", 1), ("b", 1)], [("a", 18), ("b", 1)],
         [("b", 1), ("c", 37)], [("b", 65), ("c", 2)], [("c", 1)]]


def _steps():
    at = {k: 0 for k in REQS}
    for step in STEPS:
        yield [(r, n, at[r]) for r, n in step]
        for r, n in step:
            at[r] += n
    assert at == {k: v[1] for k, v in REQS.items()}


@pytest.mark.gpu
@pytest.mark.parametrize("H,taps", [(200, 3), (45, 2), (1036, 4), (64, 1), (72, 7), (2052, 3)])
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_boundary_and_convolution_hip(H, taps, out_dtype):
    """Two sublayers in a row (a mixer's, then a feed-forward's with routed rows, a shared expert and the average over depth),
    over steps of every shape; rings filled with garbage beforehand."""
    K, dev, eps, top, slots = _K(), "cuda", 1e-5, 2, 4
    f = lambda t: t.float().to(dev).contiguous()
    w1, w2, c1, c2 = rnd(H, seed=1, std=0.2), rnd(H, seed=2, std=0.2), rnd(H, taps, seed=3), rnd(H, taps, seed=4)
    coef = torch.tensor([0.3, -0.2, 0.9], dtype=F64)
    X0, X1 = ({r: rnd(n, H, seed=s0 + i) for i, (r, (_, n)) in enumerate(REQS.items())} for s0 in (10, 20))
    Y, YB, E0, E1 = ({r: rnd(n, H, seed=s0 + i, std=0.7) for i, (r, (_, n)) in enumerate(REQS.items())} for s0 in (30, 40, 50, 60))
    mid = {r: X1[r] + Y[r] for r in REQS}
    res = {r: mid[r] + YB[r] + 0.5 * (E0[r] + E1[r]) for r in REQS}
    nxt = {r: coef[0] * X0[r] + coef[1] * X1[r] + coef[2] * res[r] for r in REQS}
    ref_mid = {r: O.input_conv(O.rms(mid[r], eps, 1.0 + w2), c2) for r in REQS}
    ref_nxt = {r: O.input_conv(O.rms(nxt[r], eps, 1.0 + w1), c1) for r in REQS}
    ref_in = {r: O.input_conv(O.rms(X1[r], eps, 1.0 + w1), c1) for r in REQS}
    ring = lambda: torch.full((slots, taps - 1, H), 7.0, device=dev) if taps > 1 else None
    r_in, r_mid, r_nxt = ring(), ring(), ring()
    tw1, tw2 = f(c1.T), f(c2.T)
    tol = 3e-5 if out_dtype == torch.float32 else 1e-2
    for step in _steps():
        cat = lambda d: torch.cat([d[r][c:c + n] for r, n, c in step])
        pos, seq, *_ = _meta([(REQS[r][0], n, c) for r, n, c in step])
        T, single = pos.numel(), all(n == 1 for _, n, _ in step)
        hist = torch.stack([f(cat(X0)), f(cat(X1)), torch.zeros(T, H, device=dev)])
        rs, h, out = torch.zeros(T, device=dev), torch.zeros(T, H, device=dev), torch.zeros(T, H, device=dev, dtype=out_dtype)
        closing = (None, None)

        def join(x_in, w, taps_w, rg, **kw):
            nonlocal closing
            cw, cr = (None, None) if single or closing[1] is None else closing
            K.stream_join(out if single else None, h, x_in, kw.get("ya"), kw.get("yb"), kw.get("ey"), kw.get("pairs"), top, 1.0 / top, kw.get("hist"),
                          kw.get("navg", 0), kw.get("coef"), f(w), rs, cw, cr, taps_w if single else None, rg if single else None, pos, seq, eps)
            closing = (f(w), rg)
            if not single:
                K.canon_conv(out, h, rs, f(w), taps_w, rg, pos, seq)
            return out.clone()

        close(join(hist[1], w1, tw1, r_in), cat(ref_in), tol)
        close(join(h, w2, tw2, r_mid, ya=f(cat(Y))), cat(ref_mid), tol)
        # the token's expert rows lie anywhere in the experts' sorted buffer
        ey, perm = torch.zeros(2 * T + 5, H, device=dev), torch.randperm(2 * T + 5, generator=torch.Generator().manual_seed(T))[:2 * T]
        ey[perm.to(dev)] = f(torch.stack([cat(E0), cat(E1)], 1).reshape(2 * T, H))
        yb = torch.zeros(T, H + 4, device=dev)
        yb[:, :H] = f(cat(YB))
        close(join(h, w1, tw1, r_nxt, yb=yb[:, :H], ey=ey, pairs=perm.to(device=dev, dtype=torch.int32), hist=hist, navg=2, coef=f(coef)), cat(ref_nxt), tol)
        close(hist[2], cat(res), 3e-6)
        close(h, cat(nxt), 3e-6)
        # the end of the stack: no norm follows, the last sublayer's inputs are saved
        K.stream_join(None, h, h, None, None, None, None, 1, 1.0, None, 0, None, None, rs, None if single or closing[1] is None else closing[0],
                      None if single else closing[1], None, None, pos, seq, eps)


LA_SIZES = [(2, 48, 32), (1, 7, 9), (3, 64, 64), (2, 130, 200), (1, 500, 44), (2, 20, 300), (1, 16, 512), (4, 128, 128), (1, 1, 1)]


@pytest.mark.gpu
@pytest.mark.parametrize("H,d,dv", LA_SIZES)
@pytest.mark.parametrize("decays", ["head", "slow", "mixed", "strong"])
def test_linear_attention_hip(H, d, dv, decays):
    """Decays per head (1, 0 and in between) and per key channel: close to one over the whole sequence, of every strength at once, so
    strong that a score tile is summed pair by pair. Steps of every shape, states full of garbage beforehand."""
    K, dev, eps, rank, slots = _K(), "cuda", 1e-5, 5, 4
    f = lambda t: t.float().to(dev).contiguous()
    head = decays == "head"
    tau = {"head": 1.0, "slow": 64.0, "mixed": 2.0, "strong": 1.0}[decays]
    qn, vn = H * d, H * dv
    cols = 2 * qn + 2 * vn + (0 if head else rank) + 3
    Z = {r: rnd(n, cols, seed=10 + i) for i, (r, (_, n)) in enumerate(REQS.items())}
    a2 = rnd(qn, rank, seed=5, std={"slow": 1.0, "mixed": 4.0, "strong": 1.0}.get(decays, 1.0))
    ab = rnd(qn, seed=6) + {"slow": 2.0, "mixed": 0.0, "strong": -6.0}.get(decays, 0.0)
    if decays == "strong":
        ab[::3] += 8.0                                    # (some channels remember, so that the outputs are not the last token's alone)
    w = 1.0 + rnd(dv, seed=7, std=0.2)
    dec = torch.tensor([(1.0, 0.0, 0.9, 0.999)[(h + d) % 4] for h in range(H)], dtype=F64)
    ref = {}
    for r, z in Z.items():
        n = z.shape[0]
        q, k, v = z[:, :qn].reshape(n, H, d) * d ** -0.5, z[:, qn:2 * qn].reshape(n, H, d), z[:, 2 * qn:2 * qn + vn].reshape(n, H, dv)
        g, low = z[:, 2 * qn + vn:2 * qn + 2 * vn], z[:, 2 * qn + 2 * vn:2 * qn + 2 * vn + rank]
        ld = torch.log(dec).view(1, H, 1).expand(n, H, d) if head else (torch.nn.functional.logsigmoid(low @ a2.T + ab) / tau).view(n, H, d)
        ref[r] = O.rms(O.linear_attention(q, k, v, ld), eps, w).reshape(n, vn) * O.silu(g)
    state = torch.full((slots, H, d, dv), 9.0, device=dev)
    hd = f(torch.stack([dec, torch.log2(dec)])) if head else None
    ws = torch.empty(int(K.linear_attention_ws_floats(128, 4, H, d, dv, not head)), device=dev)
    for dt, tol in ((torch.float32, 1e-4), (torch.bfloat16, 2e-2)):
        for step in _steps():
            z = torch.cat([Z[r][c:c + n] for r, n, c in step])
            pos, seq, qs, ctx, sl = _meta([(REQS[r][0], n, c) for r, n, c in step])
            out = torch.zeros(z.shape[0], vn, device=dev, dtype=dt)
            K.linear_attention(out, f(z), state, hd, None if head else f(a2.T), None if head else f(ab), f(w), qs, ctx, sl, H, d, dv, 0, qn, 2 * qn,
                               2 * qn + vn, 2 * qn + 2 * vn if not head else 0, d ** -0.5, 1.0 / tau, eps, max(n for _, n, _ in step), ws)
            close(out, torch.cat([ref[r][c:c + n] for r, n, c in step]), tol)
    # without a weight, a long prompt in one step (several chunks), then one more token
    n = 200
    z = rnd(n + 1, cols, seed=99)
    q, k, v = z[:, :qn].reshape(-1, H, d) * d ** -0.5, z[:, qn:2 * qn].reshape(-1, H, d), z[:, 2 * qn:2 * qn + vn].reshape(-1, H, dv)
    low = z[:, 2 * qn + 2 * vn:2 * qn + 2 * vn + rank]
    ld = torch.log(dec).view(1, H, 1).expand(n + 1, H, d) if head else (torch.nn.functional.logsigmoid(low @ a2.T + ab) / tau).view(n + 1, H, d)
    want = O.rms(O.linear_attention(q, k, v, ld), eps).reshape(n + 1, vn) * O.silu(z[:, 2 * qn + vn:2 * qn + 2 * vn])
    ws = torch.empty(int(K.linear_attention_ws_floats(n, 1, H, d, dv, not head)), device=dev)
    for lo, hi in ((0, n), (n, n + 1)):
        pos, seq, qs, ctx, sl = _meta([(3, hi - lo, lo)])
        out = torch.zeros(hi - lo, vn, device=dev)
        K.linear_attention(out, f(z[lo:hi]), state, hd, None if head else f(a2.T), None if head else f(ab), None, qs, ctx, sl, H, d, dv, 0, qn, 2 * qn,
                           2 * qn + vn, 2 * qn + 2 * vn if not head else 0, d ** -0.5, 1.0 / tau, eps, hi - lo, ws)
        close(out, want[lo:hi], 1e-4)


def _blocks(n_blocks, seed):
    return torch.randperm(n_blocks, generator=torch.Generator().manual_seed(seed))


LATENT_SIZES = [(40, 32, 4), (16, 16, 3), (128, 96, 16), (160, 128, 5), (256, 256, 2), (392, 376, 7), (512, 448, 16), (576, 512, 40), (520, 456, 1)]


@pytest.mark.gpu
@pytest.mark.parametrize("D,R,H", LATENT_SIZES)
@pytest.mark.parametrize("window", [0, 1, 33, 100])
def test_latent_attention_hip(D, R, H, window):
    """Both matrix-core kernels that read latent rows against plain softmax attention, over a paged cache whose blocks are in no
    order: prompts, portions that start anywhere, single tokens, two sequences in a step; one key at the window's far edge stands
    out for some query, one just outside for another."""
    K, dev = _K(), "cuda"
    L = {0: 150, 1: 97}                          # slot -> tokens
    bf = lambda t: t.to(torch.bfloat16)
    rows = {s: rnd(n, D, seed=3 + s) for s, n in L.items()}
    qs = {s: rnd(n, H, D, seed=5 + s) for s, n in L.items()}
    for s, n in L.items():                       # stand-out keys
        for i in (n - 1, n // 2):
            for j in ((i - window + 1, i - window) if window else (0, i // 2)):
                if 0 <= j < n:
                    rows[s][j] = rows[s][j] + 0.6 * qs[s][i, 0]
    rows, qs = {s: bf(t) for s, t in rows.items()}, {s: bf(t) for s, t in qs.items()}
    scale = 1.5 * D ** -0.5
    ref = {}
    for s, n in L.items():
        k, q = rows[s].to(F64), qs[s].to(F64)
        sc = (torch.einsum("ihd,jd->hij", q, k) * scale).masked_fill(~O.window_mask(n, window), float("-inf"))
        ref[s] = torch.einsum("hij,jd->ihd", torch.softmax(sc, -1), k[:, :R]).reshape(n, H * R)
    nb = 12
    perm = _blocks(nb, 8).tolist()
    table = torch.full((3, 6), -1, dtype=torch.int32)
    kc, vt = torch.zeros(nb, 1, 32, D, dtype=torch.bfloat16), torch.zeros(nb, 1, R, 32, dtype=torch.bfloat16)
    for s, n in L.items():
        for b in range((n + 31) // 32):
            table[s, b] = perm.pop()
        for j in range(n):
            kc[table[s, j // 32], 0, j % 32] = rows[s][j]
            vt[table[s, j // 32], 0, :, j % 32] = rows[s][j, :R]
    kc, vt, table = kc.to(dev), vt.to(dev), table.to(dev)
    part = torch.empty(max(int(K.latent_attention_part_floats(300, 2, H, R)), int(K.tile_attention_part_floats(2, H, 1, R, 1))), device=dev)
    for step in ([(0, 150, 0), (1, 97, 0)], [(1, 60, 37), (0, 2, 100)], [(0, 1, 149), (1, 1, 33)], [(0, 33, 31)], [(1, 1, 96)], [(0, 1, 0)], [(1, 1, 96), (0, 5, 64)]):
        _, _, q_start, ctx, slots = _meta(step)
        T, mq = sum(n for _, n, _ in step), max(n for _, n, _ in step)
        q = torch.cat([qs[s][c:c + n] for s, n, c in step]).reshape(T, H * D).to(dev).contiguous()
        want = torch.cat([ref[s][c:c + n] for s, n, c in step])
        for p in (part, None):                   # with and without the workspace of the key splits
            out = torch.zeros(T, H * R, device=dev, dtype=torch.bfloat16)
            K.latent_attention(out, q, kc, vt, q_start, ctx, slots, table, mq, H, scale, window, p)
            close(out, want, 1.5e-2)
        out = torch.zeros(T, H * R, device=dev, dtype=torch.bfloat16)
        K.tile_attention(out, q, D, kc, vt, q_start, ctx, slots, table, mq, H, D, R, 1, scale, window, 0, 0.0, 0.0, 1.0, 1e-5, None, part)
        close(out, want, 1.5e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("R,dr,H,d,base", [(24, 8, 3, 16, 100.0), (300, 64, 2, 10, 500000.0), (14, 6, 1, 4, 7.0)])
def test_latent_rows_into_the_cache_hip(dtype, R, dr, H, d, base):
    """The latent normed with its weight, the rotated key part and the queries' rotated parts, written through the block table; the
    queries alone for a layer that reads another layer's rows."""
    from distributed_llm_inference_amd.models.rope import rope_table
    K, dev, eps, T, c0 = _K(), "cuda", 1e-6, 45, 17
    z, w = rnd(T, H * (d + dr) + R + dr, seed=1), 1.0 + rnd(R, seed=2, std=0.3)
    pos = torch.arange(c0, c0 + T)
    hq = H * (d + dr)
    q = z[:, :hq].reshape(T, H, d + dr)
    qr = torch.cat([q[..., :d], O.rotate_pairs(q[..., d:], pos, dr, base)], -1).reshape(T, hq)
    row = torch.cat([O.rms(z[:, hq:hq + R], eps, w), O.rotate_pairs(z[:, hq + R:], pos, dr, base)], -1)
    cos, sin = (t.to(dev).contiguous() for t in rope_table(dr, base, None, 100))
    tp, ts, *_ = _meta([(1, T, c0)])
    table = torch.full((2, 4), -1, dtype=torch.int32)
    table[1] = torch.tensor([3, 0, 2, 1], dtype=torch.int32)
    table = table.to(dev)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for v_t in (True, False):
        zz = z.float().to(dev).contiguous()
        kc, vc = torch.zeros(4, 1, 32, R + dr, device=dev, dtype=dtype), torch.zeros(4, 1, R, 32, device=dev, dtype=dtype) if v_t else None
        q_out = torch.zeros(T, hq, device=dev, dtype=dtype)
        K.rope_cache_write(zz, H, d + dr, d, q_out, hq, zz[:, hq:], R + dr, 1, R + dr, R, 0, R if v_t else 0, v_t, kc, vc, dr, True, cos, sin, tp, ts,
                           table, w.float().to(dev), eps)
        close(q_out, qr, tol)
        blk = table[1].cpu().long()[pos // 32]
        close(kc.cpu()[blk, 0, pos % 32], row, tol)
        if v_t:
            close(vc.cpu()[blk, 0, :, pos % 32], row[:, :R], tol)
    zz, q_out = z.float().to(dev).contiguous(), torch.zeros(T, hq, device=dev, dtype=dtype)
    K.rope_rows(zz, H, d + dr, d, q_out, dr, True, cos, sin, tp)
    close(q_out, qr, tol)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,ff,experts,top,T", [(40, 24, 5, 2, 33), (64, 32, 3, 3, 7), (36, 10, 1, 1, 20), (128, 64, 8, 2, 700), (24, 16, 40, 4, 50)])
def test_experts_by_token_id_hip(dtype, H, ff, experts, top, T):
    """The plans of two routed layers of unequal shape in one launch, the experts' products, the weighted sum in the boundary kernel,
    the shared expert behind its sigmoid gate; limits that clip."""
    K, dev, vocab, limit, eps = _K(), "cuda", 23, 0.8, 1e-5
    ids = torch.randint(0, vocab, (T,), generator=torch.Generator().manual_seed(1))
    x, P = rnd(T, H, seed=2), {}
    for j in range(experts):
        for n, a, b in (("gate", ff, H), ("up", ff, H), ("down", H, ff)):
            P[f"e{j}.{n}"] = rnd(a, b, seed=10 + 3 * j + len(n), std=1.5 * b ** -0.5)
    for n, a, b in (("gate", ff + 4, H), ("up", ff + 4, H), ("down", H, ff + 4)):
        P["shared." + n] = rnd(a, b, seed=1000 + len(n), std=1.5 * b ** -0.5)
    P["shared.sg"] = rnd(1, H, seed=2000, std=2.0 * H ** -0.5)
    g = torch.Generator().manual_seed(3)
    P["table"] = torch.argsort(torch.rand(vocab, experts, generator=g), dim=-1)[:, :top].to(torch.int32)
    other = torch.argsort(torch.rand(vocab, 6, generator=g), dim=-1)[:, :3].to(torch.int32)
    if dtype == torch.bfloat16:
        x = x.to(dtype).to(F64)
        P = {k: (v.to(dtype).to(F64) if v.is_floating_point() else v) for k, v in P.items()}
    ref = O.moe_ff(x, P, {"router": {"top": top}, "expert": {"limit": limit}, "shared": {"limit": 1.3}}, ids.tolist())
    d = lambda t: t.to(device=dev, dtype=dtype).contiguous()
    big = dtype == torch.bfloat16 and H % 32 == 0 and ff % 32 == 0
    shapes = [(3, 6, False), (top, experts, big)]
    tables = torch.cat([other.reshape(-1), P["table"].reshape(-1)]).to(dev)
    desc, off, at = [], 0, [0, 0, 0]
    for tp, ex, bg in shapes:
        tr = 128 if bg and T * tp >= 1024 else 32
        nt = (T * tp + tr - 1) // tr + ex
        desc.append([off, tp, ex, at[0], at[1], at[2], int(bg), 0])
        off, at = off + vocab * tp, [at[0] + 1 + nt, at[1] + nt * tr, at[2] + T * tp]
    host = torch.tensor(desc, dtype=torch.int32)
    tiles, row_tok, pair_row = (torch.full((n,), 77777, dtype=torch.int32, device=dev) for n in at)
    K.moe_table_plan(tiles, row_tok, pair_row, tables, ids.to(device=dev, dtype=torch.int32), host.to(dev), host, T, vocab, 1024)
    # the first layer's plan: every pair has a row of its own in a tile of its expert
    pr = pair_row[:3 * T].cpu().reshape(T, 3)
    assert pr.unique().numel() == 3 * T
    for t in range(T):
        for i in range(3):
            r = int(pr[t, i])
            assert int(row_tok[r]) == t and int(tiles[1 + r // 32]) == int(other[ids[t], i])
    _, tp, ex, ot, orow, op, bg, _ = desc[1]
    eact, ey = torch.zeros(tr * nt, ff, device=dev, dtype=dtype), torch.zeros(tr * nt, H, device=dev)
    stack = lambda n: d(torch.stack([P[f"e{j}.{n}"] for j in range(experts)]))
    K.moe_up(eact, d(x), stack("gate"), stack("up"), tiles[ot:], row_tok[orow:], nt, limit, tr)
    K.moe_down(ey, eact, stack("down"), tiles[ot:], row_tok[orow:], nt, tr)
    z = torch.cat([x @ P["shared.gate"].T, x @ P["shared.up"].T, x @ P["shared.sg"].T, torch.zeros(T, 3, dtype=F64)], 1).float().to(dev)
    acts = torch.zeros(T, ff + 4, device=dev, dtype=dtype)
    K.glu_act(acts, z, 1.3, True)
    yb = acts.float() @ P["shared.down"].float().to(dev).T
    h, rs = torch.zeros(T, H, device=dev), torch.zeros(T, device=dev)
    pos, seq, *_ = _meta([(0, T, 0)])
    K.stream_join(None, h, torch.zeros(T, H, device=dev), None, yb.contiguous(), ey, pair_row[op:], top, 1.0 / top, None, 0, None, None, rs, None, None,
                  None, None, pos, seq, eps)
    close(h, ref, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("F", [33, 40, 3000])
def test_polynomial_hip(dtype, F):
    K, dev = _K(), "cuda"
    z, c = rnd(11, F + 4, seed=1, std=2.0), torch.tensor([0.5, -0.3, 0.7, 0.2], dtype=F64)
    out = torch.zeros(11, F, device=dev, dtype=dtype)
    K.poly_norm(out, z.float().to(dev), c.float().to(dev), 1e-5)
    close(out, O.poly_norm(z[:, :F], 1e-5, c), 1e-5 if dtype == torch.float32 else 1e-2)
