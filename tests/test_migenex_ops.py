"""Every mechanism of the Migenex design alone: the package's torch operations (CPU) and its HIP kernels (`gpu` marker)
against the plain float64 functions of `migenex_oracle`, on small inputs made here."""
import pytest
import torch

import migenex_oracle as O

F64 = torch.float64


def rnd(*shape, seed=0, std=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64) * std


def close(got, ref, tol=2e-5):
    ref = ref.to(F64)
    err = (got.detach().cpu().to(F64) - ref).abs().max().item() / max(1.0, ref.abs().max().item())
    assert err < tol, err


# ---- torch operations (the CPU executor's) ---------------------------------------------------------------------------
@pytest.mark.parametrize("d,dims,base", [(14, 14, 100.0), (14, 6, 500000.0), (8, 2, 7.0)])
def test_rotations(d, dims, base):
    from distributed_llm_inference_amd.models.rope import rope_table
    from distributed_llm_inference_amd.ops import reference as R
    x, pos = rnd(6, 2, d, seed=6), torch.tensor([0, 1, 2, 50, 700, 703])
    cos, sin = rope_table(dims, base, None, 710)
    close(R.rope_partial(x.float(), cos, sin, pos, True), O.rotate_pairs(x, pos, dims, base), 1e-5)
    close(R.rope_partial(x.float(), cos, sin, pos, False), O.rotate_halves(x, pos, dims, base), 1e-5)


@pytest.mark.parametrize("window,cap", [(0, 2.0), (1, 0.0), (7, 0.0), (33, 5.0)])
def test_attention(window, cap):
    from distributed_llm_inference_amd.ops import reference as R
    q, k, v = rnd(60, 4, 8, seed=7, std=2.0), rnd(60, 2, 8, seed=8), rnd(60, 2, 5, seed=9)
    ref = O.softmax_attention(q, k, v, 0.7, O.visible(60, window), cap)
    got = torch.cat([R.attention(q[a:b].float(), k[:b].float(), v[:b].float(), a, 0.7, window=window, softcap=cap) for a, b in ((0, 31), (31, 33), (33, 60))])
    close(got.reshape(60, -1), ref)


@pytest.mark.parametrize("top", [1, 2, 5])
def test_routing(top):
    from distributed_llm_inference_amd.ops import reference as R
    z = rnd(40, 5, seed=1)
    idx, w = R.moe_route(torch.sigmoid(z.float()), top, 1, 1, 1.0, group_rank=1, renorm=False)
    s = torch.sigmoid(z)
    assert torch.equal(idx, torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top])
    close(w, s.gather(1, idx))


def test_weight_on_the_input_is_a_factor_of_the_products():
    """up(w h) = w up(h): what the executors use; the activation makes it differ from a weight on the output."""
    h, P = rnd(9, 12, seed=1), {"e0.up": rnd(20, 12, seed=2), "e0.down": rnd(12, 20, seed=3)}
    w = torch.sigmoid(rnd(9, 1, seed=4))
    want = O.expert(w * h, P, "e0.")
    close(torch.relu(w * (h @ P["e0.up"].T)) ** 2 @ P["e0.down"].T, want, 1e-12)
    assert (w * O.expert(h, P, "e0.") - want).abs().max() > 0.1 * want.abs().max()


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


def _table(lengths, rows, cols, n_blocks, seed):
    """A block table whose blocks are in no order; rows without a sequence hold -1."""
    perm = torch.randperm(n_blocks, generator=torch.Generator().manual_seed(seed)).tolist()
    table = torch.full((rows, cols), -1, dtype=torch.int32)
    for s, n in lengths.items():
        for b in range((n + 31) // 32):
            table[s, b] = perm.pop()
    return table


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,buckets,mp,mc", [(40, 53, 7, 11), (33, 1, 0, 1), (200, 65521, 2147483629, 2147483587)])
def test_embedding_hip(dtype, H, buckets, mp, mc):
    """Portions of every size, requests that pause, pages full of garbage and used by another request before; both halves of the pass
    map's rows."""
    K, dev, vocab, scale = _K(), "cuda", 1000, 2.5
    W = {"embed": rnd(vocab, H, seed=1).to(dtype), "bigram": rnd(min(buckets, 70000) + 1, H, seed=2).to(dtype)}
    cfg = {"embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mp, "mul_cur": mc}}}
    g = torch.Generator().manual_seed(3)
    reqs = {s: torch.randint(0, vocab, (n,), generator=g).tolist() for s, n in ((2, 70), (0, 40))}
    ref = {s: O.embedding(cfg, W, t) for s, t in reqs.items()}
    table = _table({2: 70, 0: 40}, 4, 3, 6, 4).to(dev)
    pages = torch.full((6, 32), 7, dtype=torch.int32, device=dev)
    emb, big = W["embed"].to(dev), W["bigram"].to(dev)
    for step in ([(2, 32, 0)], [(0, 2, 0), (2, 1, 32)], [(2, 2, 33), (0, 30, 2)], [(0, 1, 32)], [(2, 1, 35), (0, 1, 33)], [(2, 34, 36), (0, 6, 34)], [(3, 1, 0), (3, 1, 5)]):
        pos, seq, *_ = _meta(step)
        T = pos.numel()
        toks = [reqs[s][c + i] if s in reqs else 5 for s, n, c in step for i in range(n)]
        ids = torch.tensor(toks, dtype=torch.int32, device=dev)
        out, cat = torch.zeros(T, H, device=dev), torch.full((T, 2 * H), 9.0, device=dev, dtype=dtype)
        K.embed_bigram(out, cat, False, ids, emb, scale, big, mp, mc, pages, pos, seq, table)
        if step[0][0] == 3:                          # rows without blocks (padding of a fixed-shape step): nothing is written
            assert torch.equal(pages, before)
            continue
        before = pages.clone()
        want = torch.cat([ref[s][c:c + n] for s, n, c in step])
        close(out, want, 1e-6)
        close(cat[:, H:], want, 1e-6 if dtype == torch.float32 else 5e-3)
        assert (cat[:, :H] == 9.0).all()
        K.embed_bigram(out, cat, True, ids, emb, scale, big, mp, mc, pages, pos, seq, table)       # (a step that runs twice)
        close(out, want, 1e-6)
        assert torch.equal(cat[:, :H], cat[:, H:])
    out = torch.zeros(4, H, device=dev)
    K.embed_bigram(out, None, False, torch.tensor([1, 2, -5, vocab + 3], dtype=torch.int32, device=dev), emb, scale, None, 0, 0, None, *_meta([(2, 4, 0)])[:2], table)
    close(out, W["embed"].to(F64)[[1, 2, 0, vocab - 1]] * scale, 1e-6)


@pytest.mark.gpu
@pytest.mark.parametrize("H", [37, 48, 200, 1036, 2048, 3001, 8192])
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_boundary_hip(H, out_dtype):
    """Every use of the boundary kernel: a GEMM's output whole or in partial sums, alone and with routed rows in any order, before a norm, before
    the pass map (the stream itself, into half of wider rows), at the end, and the norm alone."""
    K, dev, T, eps, top = _K(), "cuda", 9, 1e-5, 2
    f = lambda t: t.float().to(dev).contiguous()
    x, ya, yb, E = rnd(T, H, seed=1), rnd(T, H, seed=2, std=3.0), rnd(T, H, seed=3), rnd(T, top, H, seed=4)
    wb, wn = 0.5 * (1.0 + rnd(H, seed=5, std=0.2)), 1.0 + rnd(H, seed=6, std=0.2)
    pad = torch.zeros(T, H + 4, device=dev)
    perm = torch.randperm(3 * T, generator=torch.Generator().manual_seed(7))[:top * T]
    ey = torch.full((3 * T, H), 1e3, device=dev)
    ey[perm.to(dev)] = f(E.reshape(top * T, H))
    pairs = perm.to(device=dev, dtype=torch.int32).clone()
    pairs[3] = -1                                      # (a choice without a row)
    E2 = E.clone()
    E2[1, 1] = 0.0
    tol = 2e-5 if out_dtype == torch.float32 else 1e-2
    parts = torch.zeros(5, T + 2, H + 4, device=dev)
    parts[:, :T, :H] = f(torch.stack([rnd(T, H, seed=20 + i) for i in range(5)]))
    psum = sum(rnd(T, H, seed=20 + i) for i in range(5))
    pad[:, :H] = f(ya)
    for a, given, e in ((ya, pad[:, :H], None), (yb, f(yb), E2), (None, None, E2), (psum, parts[:, :, :H], None), (psum, parts[:, :, :H], E2)):
        y = sum(t for t in (a, e.sum(1) if e is not None else None) if t is not None)
        want = x + O.rms(y, eps, wb)
        args = (given, ey if e is not None else None, pairs if e is not None else None, top, f(wb))
        h, out = f(x), torch.zeros(T, H, device=dev, dtype=out_dtype)
        K.sandwich_join(out, h, *args, f(wn), eps)
        close(h, want)
        close(out, O.rms(want, eps, wn), tol)
        h, cat = f(x), torch.full((T, 2 * H), 5.0, device=dev, dtype=out_dtype)
        K.sandwich_join(cat[:, :H], h, *args, None, eps)
        close(h, want)
        close(cat[:, :H], want, tol)
        assert (cat[:, H:] == 5.0).all()
        h = f(x)
        K.sandwich_join(None, h, *args, None, eps)
        close(h, want)
    h, out = f(x), torch.zeros(T, H, device=dev, dtype=out_dtype)
    K.sandwich_join(out, h, None, None, None, 1, None, f(wn), eps)
    close(out, O.rms(x, eps, wn), tol)
    assert torch.equal(h, f(x))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("F", [33, 40, 3000])
def test_activations_hip(dtype, F):
    K, dev = _K(), "cuda"
    z = rnd(11, 2 * F + 8, seed=1, std=2.0)
    for zt in (torch.float32, torch.bfloat16):
        zz, out = z.to(device=dev, dtype=zt), torch.zeros(11, F, device=dev, dtype=dtype)
        zr, tol = zz.cpu().to(F64), 1e-6 if dtype == torch.float32 else 5e-3
        K.relu_act(out, zz[:, 3:3 + F], False)
        close(out, torch.relu(zr[:, 3:3 + F]) ** 2, tol)
        K.relu_act(out, zz, True)
        close(out, torch.relu(zr[:, :F]) * zr[:, F:2 * F], tol)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,ff,experts,top,T", [(40, 24, 5, 2, 33), (64, 32, 3, 3, 7), (36, 10, 1, 1, 20), (128, 64, 8, 2, 700), (96, 160, 6, 1, 1100), (24, 16, 40, 4, 50)])
def test_routed_feed_forward_hip(dtype, H, ff, experts, top, T):
    """route -> plan with the weights at the rows -> the gateless experts on weighted inputs -> sum in the boundary kernel, with a
    shared expert; both tile sizes; buffers full of garbage beforehand."""
    K, dev, eps = _K(), "cuda", 1e-5
    x, P = rnd(T, H, seed=2), {"router": rnd(experts, H, seed=3, std=2.0 * H ** -0.5), "shared.up": rnd(ff + 4, H, seed=4, std=H ** -0.5),
                               "shared.down": rnd(H, ff + 4, seed=5, std=ff ** -0.5)}
    for j in range(experts):
        P[f"e{j}.up"], P[f"e{j}.down"] = rnd(ff, H, seed=10 + 2 * j, std=1.5 * H ** -0.5), rnd(H, ff, seed=11 + 2 * j, std=1.5 * ff ** -0.5)
    if dtype == torch.bfloat16:
        x, P = x.to(dtype).to(F64), {k: v.to(dtype).to(F64) for k, v in P.items()}
    ref = O.routed_ff(x, P, {"router": {"top": top}, "shared": {"ff": ff + 4}})
    d = lambda t: t.to(device=dev, dtype=dtype).contiguous()
    f = lambda t: t.float().to(dev).contiguous()
    tr = 128 if dtype == torch.bfloat16 and H % 32 == 0 and ff % 32 == 0 and T * top >= 1024 else 32
    nt = (T * top + tr - 1) // tr + experts
    sel, wts = torch.zeros(T * top, dtype=torch.int32, device=dev), torch.zeros(T * top, device=dev)
    z = f(x @ P["router"].T)
    K.moe_route(sel, wts, z, top, 1, 1, 1.0, None, False, 1, False)
    tiles, row_tok, pair_row = (torch.full((n,), 77777, dtype=torch.int32, device=dev) for n in (1 + nt, tr * nt, T * top))
    row_w = torch.full((tr * nt,), float("nan"), device=dev)
    K.moe_plan(tiles, row_tok, pair_row, sel, T * top, top, experts, tr, wts, row_w)
    # both in one call: the same choices and weights, every pair in a row of its own in a tile of its expert
    again = [torch.full_like(t, 7) for t in (sel, wts, tiles, row_tok, pair_row, row_w)]
    K.moe_route_plan(again[0], again[1], z, top, 1, 1, 1.0, None, False, 1, False, again[2], again[3], again[4], experts, tr, again[5])
    assert torch.equal(again[0], sel) and torch.equal(again[1], wts) and torch.equal(again[2][:1 + int(tiles[0])], tiles[:1 + int(tiles[0])])
    pr = again[4].cpu().long()
    assert pr.unique().numel() == T * top and torch.equal(again[2].cpu()[1 + pr // tr], sel.cpu()) and torch.equal(again[5].cpu()[pr], wts.cpu())
    assert torch.equal(again[3].cpu()[pr], torch.arange(T * top, dtype=torch.int32) // top)
    pr = pair_row.cpu().long()
    assert pr.unique().numel() == T * top and torch.equal(row_w.cpu()[pr], wts.cpu())
    eact, ey = torch.full((tr * nt, ff), 3.0, device=dev, dtype=dtype), torch.full((tr * nt, H), 3.0, device=dev)
    stack = lambda n: d(torch.stack([P[f"e{j}.{n}"] for j in range(experts)]))
    K.moe_up(eact, d(x), None, stack("up"), tiles, row_tok, nt, 0.0, tr, row_w)
    K.moe_down(ey, eact, stack("down"), tiles, row_tok, nt, tr)
    act = torch.zeros(T, ff + 4, device=dev, dtype=dtype)
    K.relu_act(act, f(x @ P["shared.up"].T), False)
    yb = (act.float() @ P["shared.down"].float().to(dev).T).contiguous()
    h = torch.zeros(T, H, device=dev)
    K.sandwich_join(None, h, yb, ey, pair_row, top, torch.ones(H, device=dev), None, eps)
    close(h, O.rms(ref, eps), 3e-5 if dtype == torch.float32 else 2e-2)


PREP = [(4, 2, 16, 24, 16, False, "norm"), (3, 1, 12, 70, 6, True, "norm"), (5, 5, 7, 7, 2, False, "both"), (6, 2, 64, 64, 64, True, "unit"),
        (8, 2, 128, 128, 32, False, "norm"), (4, 4, 96, 96, 96, True, "unit"), (2, 1, 160, 160, 80, True, "unit"), (1, 1, 300, 44, 300, False, "norm"),
        (3, 3, 65, 65, 0, True, "unit"), (16, 1, 8, 8, 8, True, "unit"), (2, 2, 512, 512, 512, False, "norm")]


@pytest.mark.gpu
@pytest.mark.parametrize("layout", ["rows", "tiles", "fragments"])
@pytest.mark.parametrize("keyed", [False, True])
@pytest.mark.parametrize("H,G,d,dv,dims,inter,norms", PREP)
def test_query_key_preparation_hip(H, G, d, dv, dims, inter, norms, keyed, layout):
    """Norms ahead of and behind the rotation, both pairings, rotated parts, values of their own or the keys as projected, every cache
    layout, 32-bit and bf16 in and out."""
    from distributed_llm_inference_amd.models.rope import rope_table
    if (keyed and dv != d) or (layout == "fragments" and not (d == dv and d in (64, 128))):
        pytest.skip("a combination that does not exist")
    K, dev, eps, T, c0, base = _K(), "cuda", 1e-6, 45, 17, 300.0
    cols = (H + G) * d + (0 if keyed else G * dv)
    z_all, qw, kw = rnd(T, cols + 8, seed=1, std=1.7), 1.0 + rnd(d, seed=2, std=0.3), 1.0 + rnd(d, seed=3, std=0.3)
    pos = torch.arange(c0, c0 + T)
    cos, sin = (t.to(dev).contiguous() for t in rope_table(dims, base, None, 100)) if dims else (None, None)
    tp, ts, *_ = _meta([(1, T, c0)])
    table = torch.full((2, 4), -1, dtype=torch.int32)
    table[1] = torch.tensor([3, 0, 2, 1], dtype=torch.int32)
    blk, off = table[1].long()[pos // 32], pos % 32
    table = table.to(dev)
    f = lambda t: t.float().to(dev).contiguous()
    nw = norms in ("norm", "both")
    for zt, qt, ct in ((torch.float32,) * 3, (torch.float32, torch.float32, torch.bfloat16), (torch.float32, torch.bfloat16, torch.bfloat16), (torch.bfloat16,) * 3):
        if layout == "fragments" and ct != torch.bfloat16:
            continue
        z = z_all.to(zt)
        zr = z.to(F64)
        q, k = zr[:, :H * d].reshape(T, H, d), zr[:, H * d:(H + G) * d].reshape(T, G, d)
        v = k if keyed else zr[:, (H + G) * d:cols].reshape(T, G, dv)
        if nw:
            q, k = O.rms(q, eps, qw), O.rms(k, eps, kw)
        turn = O.rotate_pairs if inter else O.rotate_halves
        q, k = turn(q, pos, dims, base), turn(k, pos, dims, base)
        if norms in ("unit", "both"):
            q, k = O.rms(q, eps), O.rms(k, eps)
        q_out = torch.zeros(T, H * d, device=dev, dtype=qt)
        zeros = lambda *s: torch.zeros(*s, device=dev, dtype=ct)
        kc = zeros(4, G, 2, 32 * d) if layout == "fragments" else zeros(4, G, 32, d)
        vc = None if layout == "fragments" else zeros(4, G, dv, 32) if layout == "tiles" else zeros(4, G, 32, dv)
        K.qk_prep(z.to(dev), H, G, d, dv, -1 if keyed else (H + G) * d, f(qw) if nw else None, f(kw) if nw else None, norms != "norm", eps, dims, inter,
                  cos, sin, q_out, kc, vc, {"rows": 0, "tiles": 1, "fragments": 2}[layout], tp, ts, table)
        tol = lambda t: 2e-5 if t == torch.float32 else 1e-2
        close(q_out.view(T, H, d), q, tol(qt))
        if layout == "fragments":
            kk, dd = torch.arange(32).view(32, 1), torch.arange(d).view(1, d)
            ko = (kk >> 4) * (16 * d) + ((dd >> 3) * 16 + (kk & 15)) * 8 + (dd & 7)
            vo = (((dd >> 4) * 4 + ((kk & 15) >> 2)) * 16 + (dd & 15)) * 8 + ((kk >> 4) * 4 + (kk & 3))
            slab = kc.cpu()[blk]                                        # [T, G, 2, 32 d]
            got_k = slab[:, :, 0].gather(2, ko[off].unsqueeze(1).expand(T, G, d))
            got_v = slab[:, :, 1].gather(2, vo[off].unsqueeze(1).expand(T, G, d))
        else:
            got_k = kc.cpu()[blk, :, off]
            got_v = vc.cpu()[blk, :, :, off] if layout == "tiles" else vc.cpu()[blk, :, off]
        close(got_k, k, tol(ct))
        close(got_v, v, tol(ct))
        # places outside the written positions stay as they were, and a row without blocks writes nothing
        before = kc.clone()
        K.qk_prep(z.to(dev)[:1], H, G, d, dv, -1 if keyed else (H + G) * d, None, None, True, eps, 0, inter, None, None, q_out, kc, vc,
                  {"rows": 0, "tiles": 1, "fragments": 2}[layout], tp[:1], torch.zeros(1, dtype=torch.int32, device=dev), table)
        assert torch.equal(before, kc)


@pytest.mark.gpu
@pytest.mark.parametrize("D,H,G,window,cap,gated", [(64, 4, 2, 40, 0.0, True), (64, 6, 2, 0, 3.0, False), (128, 4, 1, 33, 0.0, True), (128, 16, 1, 0, 30.0, False),
                                                    (128, 8, 2, 100, 2.0, True), (64, 3, 3, 1, 0.0, True), (64, 16, 4, 0, 1.5, True)])
def test_capped_and_gated_attention_hip(D, H, G, window, cap, gated):
    """The MFMA attention kernels with capped scores and the entry gate, over blocks in no order: prompts (the prefill-shaped kernel),
    short portions, single tokens (four waves per item, and one with many items), two sequences in a step; one key at the window's
    far edge stands out for some query, one just outside for another, one far back over the whole context."""
    K, dev = _K(), "cuda"
    L = {0: 150, 1: 97}
    bf = lambda t: t.to(torch.bfloat16)
    ks, vs, qs, gs = ({s: rnd(n, hh, D, seed=sd + s) for s, n in L.items()} for sd, hh in ((3, G), (5, G), (7, H), (9, H)))
    for s, n in L.items():
        for i in (n - 1, n // 2):
            for j in ((i - window + 1, i - window) if window else (0, i // 2)):
                if 0 <= j < n:
                    ks[s][j, 0] = ks[s][j, 0] + 0.8 * qs[s][i, 0]
    ks, vs, qs, gs = ({s: bf(t) for s, t in x.items()} for x in (ks, vs, qs, gs))
    scale = 1.5 * D ** -0.5
    ref = {}
    for s, n in L.items():
        o = O.softmax_attention(qs[s].to(F64), ks[s].to(F64), vs[s].to(F64), scale, O.visible(n, window), cap)
        ref[s] = o * torch.sigmoid(gs[s].to(F64).reshape(n, -1)) if gated else o
    table = _table(L, 3, 6, 12, 8)
    kv = torch.zeros(12, G, 2, 32 * D, dtype=torch.bfloat16)
    kk, dd = torch.arange(32).view(32, 1), torch.arange(D).view(1, D)
    ko = (kk >> 4) * (16 * D) + ((dd >> 3) * 16 + (kk & 15)) * 8 + (dd & 7)
    vo = (((dd >> 4) * 4 + ((kk & 15) >> 2)) * 16 + (dd & 15)) * 8 + ((kk >> 4) * 4 + (kk & 3))
    for s, n in L.items():
        for j in range(n):
            b = int(table[s, j // 32])
            for g in range(G):
                kv[b, g, 0, ko[j % 32]] = ks[s][j, g]
                kv[b, g, 1, vo[j % 32]] = vs[s][j, g]
    kv, table = kv.to(dev), table.to(dev)
    steps = [[(0, 150, 0), (1, 97, 0)], [(1, 60, 37), (0, 2, 100)], [(0, 1, 149), (1, 1, 33)], [(0, 33, 31)], [(1, 1, 96)], [(0, 1, 0)], [(1, 1, 96), (0, 5, 64)],
             [(0, 1, 149), (1, 1, 96)] * 600]
    for step in steps:
        _, _, q_start, ctx, slots = _meta(step)
        T, mq = sum(n for _, n, _ in step), max(n for _, n, _ in step)
        cat = lambda x: torch.cat([x[s][c:c + n].reshape(n, -1) for s, n, c in step]).to(dev).contiguous()
        wide = torch.zeros(T, H * D + 8, device=dev, dtype=torch.bfloat16)
        wide[:, 4:4 + H * D] = cat(gs)
        out = torch.zeros(T, H * D, device=dev, dtype=torch.bfloat16)
        K.paged_attention_capped(out, cat(qs), kv, q_start, ctx, table, slots, mq, H, G, D, scale, window, cap, wide[:, 4:4 + H * D] if gated else None)
        close(out, torch.cat([ref[s][c:c + n] for s, n, c in step]), 1.5e-2)
