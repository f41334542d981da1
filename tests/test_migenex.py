"""Migenex through the package (checkpoint reader, executor, cache and state slots, trace replay, scheduler) against the
plain model in `migenex_oracle`. Every test runs on the torch executor on the CPU; the same tests run on the HIP executor,
in fp32 and in bf16, under the `gpu` marker."""
import copy

import numpy as np
import pytest
import torch

from migenex_util import (SAME, STACKS, TOL, alone, dense, full, keyed, make_config, moe, oracle_logits, random_tokens, random_weights, rel_err,
                          replay, save_model, session)

BACKENDS = [pytest.param("torch", "fp32", id="torch"),
            pytest.param("hip", "fp32", id="hip-fp32", marks=pytest.mark.gpu),
            pytest.param("hip", "bf16", id="hip-bf16", marks=pytest.mark.gpu)]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for i, (name, cfg) in enumerate(STACKS.items()):
        W = random_weights(cfg, seed=60 + i)
        out[name] = (cfg, W, save_model(str(tmp_path_factory.mktemp(name)), cfg, W))
    return out


def pos_errs(got, ref):
    d = got.astype(np.float64) - ref
    d = d - d.mean(-1, keepdims=True)
    r = ref - ref.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((r ** 2).mean(-1)).mean()


def check(got, ref, dtype, what="", same_as=None, share=1.0):
    """fp32: every position. bf16: `share` of them (see `share_of`; a handful of positions is then too few to judge)."""
    share = 1.0 if dtype == "fp32" else share
    if share < 1.0 and len(got) < 10:
        return
    e = float(np.quantile(pos_errs(got, ref), share))
    assert e < TOL[dtype], f"{what}: error {e:.3g} over {TOL[dtype]}"
    if same_as is not None:
        e = float(np.quantile(pos_errs(got, same_as.astype(np.float64)), share))
        assert e < SAME[dtype], f"{what}: differs from the whole prompt run alone by {e:.3g}, over {SAME[dtype]}"


def share_of(cfg):
    """A router is a discontinuity: where two experts nearly tie, one bf16 rounding moves a whole position. Nine positions in ten then."""
    return 0.9 if any((l["mlp"] or {}).get("kind") == "moe" and l["mlp"]["router"]["experts"] > l["mlp"]["router"]["top"] for l in cfg["layers"]) else 1.0


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_whole_prompt(models, stack, backend, dtype):
    """Logits, and the stream after every layer run."""
    import migenex_oracle as O
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, 145, 1)
    sess = session(path, backend, dtype)
    sess.ex.keep_layer_outputs = True
    got = replay(sess, {"a": toks}, [[("a", len(toks))]])["a"]
    layers = [x.float().cpu().numpy() for x in sess.ex.layer_outputs]
    sess.close()
    ref, after = O.forward(cfg, W, toks)
    assert len(layers) == len(after)
    for i, (a, b) in enumerate(zip(layers, after)):
        err = np.sqrt(((a - b.numpy()) ** 2).mean()) / np.sqrt((b.numpy() ** 2).mean())
        assert err < (3e-5 if dtype == "fp32" else 0.05), f"layer {i}: {err:.3g}"
    check(got, ref.numpy(), dtype, stack, share=share_of(cfg))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_prefill_then_token_by_token(models, stack, backend, dtype):
    """A prompt, then decoding one token a step across the windows' edges of every layer and over several cache blocks."""
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, 120, 2)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", 30)]] + [[("a", 1)]] * 90)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, stack, alone(path, backend, dtype, toks), share_of(cfg))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_first_tokens_alone(models, stack, backend, dtype):
    """A sequence that starts token by token: no previous token, windows that are not full yet."""
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, 12, 3)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", 1)]] * 12)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, stack, alone(path, backend, dtype, toks), share_of(cfg))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack,cuts", [("mixed", [2, 2, 3, 1, 12, 2, 18, 33, 2, 1, 5, 31]), ("odd_sizes", [1, 2, 31, 2, 2, 36, 1, 3, 2, 34, 64, 2]),
                                        ("plain", [2] * 30), ("packed", [2, 31, 2, 1, 97, 3, 130, 2, 33]),
                                        ("packed_dense", [3, 30, 2, 2, 128, 1, 64, 2, 33])])
def test_portions(models, stack, cuts, backend, dtype):
    """Prompts cut into portions of changing size, down to two tokens, in the middle of cache blocks and windows."""
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, sum(cuts), 4)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", c)] for c in cuts])["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, stack, alone(path, backend, dtype, toks), share_of(cfg))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_mixed_batches_and_reuse(models, stack, backend, dtype):
    """Unequal requests share steps (portions beside single tokens), more requests than slots over time, a pool that only
    holds the live ones: slots and blocks change hands. Every request must come out as if it ran alone."""
    cfg, W, path = models[stack]
    reqs = {n: random_tokens(cfg, ln, 20 + i) for i, (n, ln) in enumerate([("a", 70), ("b", 9), ("c", 41), ("d", 100), ("e", 35), ("f", 66), ("g", 3)])}
    sched = [[("a", 33), ("b", 2)], [("a", 1), ("b", 7), ("c", 30)], [("a", 30), ("c", 1), ("d", 64)],
             [("a", 1), ("c", 1), ("d", 1), ("e", 35)],                      # b ended: e takes its slot; e ends at once
             [("a", 5), ("c", 9), ("d", 30), ("f", 2)], [("d", 1), ("f", 62), ("g", 1)], [("d", 2), ("f", 1), ("g", 2)],
             [("d", 2), ("f", 1)]]
    sess = session(path, backend, dtype, max_tokens=352, slots=4)
    got = replay(sess, reqs, sched)
    assert sess.alloc.used == 0 and all(r is None for r in sess.rows)
    sess.close()
    for name, toks in reqs.items():
        check(got[name], oracle_logits(cfg, W, toks), dtype, f"{stack}/{name}", alone(path, backend, dtype, toks), share_of(cfg))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
def test_slot_taken_over_starts_clean(models, backend, dtype):
    """One slot, one request after another: the second must not see the first one's tokens or cache rows."""
    cfg, W, path = models["mixed"]
    a, b = random_tokens(cfg, 50, 31), random_tokens(cfg, 20, 32)
    sess = session(path, backend, dtype, max_tokens=64, slots=1)
    got = replay(sess, {"a": a, "b": b}, [[("a", 50)], [("b", 1)], [("b", 2)], [("b", 17)]])
    sess.close()
    check(got["b"], oracle_logits(cfg, W, b), dtype, "second", alone(path, backend, dtype, b), share_of(cfg))
    check(got["a"], oracle_logits(cfg, W, a), dtype, "first", alone(path, backend, dtype, a), share_of(cfg))


def _beacon_model(kind: str, window: int):
    """One layer whose single key stands out: token 7's key is large along an entry that token 9's query asks for. No rotation, so
    that the distance alone decides whether the key is seen. A second, plain layer follows in a pass of its own."""
    att = keyed(4, 2, 16, window, rot=0, scale=1.0) if kind == "keyed" else full(4, 2, 16, 16, rot=0, scale=1.0, cap=60.0)
    cfg = make_config([att, keyed(2, 1, 8, 3, mlp=dense(16))], vocab=40, width=32, loop=(0, 1, 2), mult=1.0, scale=1.0, bigram=None)
    W = random_weights(cfg, seed=5)
    e7, e9 = W["embed"][7].float(), W["embed"][9].float()
    e9 = e9 - e7 * (e9 @ e7) / (e7 @ e7)                # (orthogonal to each other and of equal length, the others free of both)
    e9 = e9 * e7.norm() / e9.norm()
    E = W["embed"].float()
    for t in range(40):
        for u in (e7, e9):
            E[t] = E[t] - u * (E[t] @ u) / (u @ u)
    E[7], E[9] = e7, e9
    W["embed"] = E.to(torch.bfloat16)
    W["loop.in"] = torch.cat([0.05 * torch.eye(32), torch.eye(32)], 1).to(torch.bfloat16)      # (every pass reads the embedding)
    W["l0.norm1"] = torch.ones(32, dtype=torch.bfloat16)
    q, k = W["l0.mix.q"].float(), W["l0.mix.k"].float()
    for rows in (q, k):
        rows.mul_(0.3)
        for u in (e7, e9):
            rows.sub_(torch.outer(rows @ u, u) / (u @ u))
    q[::16] += 2.0 * e9 / e9.norm()                     # every head's first query entry asks, every key's first entry answers
    k[::16] += 2.0 * e7 / e7.norm()
    W["l0.mix.q"], W["l0.mix.k"] = q.to(torch.bfloat16), k.to(torch.bfloat16)
    if kind == "full":
        W["l0.mix.q.norm"], W["l0.mix.k.norm"] = torch.ones(16, dtype=torch.bfloat16), torch.ones(16, dtype=torch.bfloat16)
    return cfg, W


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("kind,window", [("keyed", 130), ("keyed", 32), ("full", 0)])
def test_window_edges_and_far_keys(tmp_path, backend, dtype, kind, window):
    """A key that stands out at the window's last place, one position outside, right behind the asking token and across cache
    blocks; in a prompt, in portions cut around the asking token, and in decoding; over the whole context as well. A window that is
    one token off moves the logits by far more than the tolerance."""
    cfg, W = _beacon_model(kind, window)
    path = save_model(str(tmp_path / "m"), cfg, W)
    base = [t for t in random_tokens(cfg, 500, 6) if t not in (7, 9)][:300]

    def placed(beacon, ask):
        toks = list(base)
        toks[beacon], toks[ask] = 7, 9
        return toks, oracle_logits(cfg, W, toks)

    w = window or 250
    for beacon, ask in [(0, w - 1), (0, w), (40, 40 + w - 1), (39, 40 + w - 1), (w, w + 1), (31, 31 + w - 1), (32, 32 + w), (299 - w, 298)]:
        toks, ref = placed(beacon, ask)
        for sched in ([[("a", 300)]], [[("a", ask - 1)], [("a", 2)]] + [[("a", 300 - ask - 1)]] * (ask < 299), [[("a", ask)]] + [[("a", 1)]] * min(3, 300 - ask)):
            n = sum(c for step in sched for _, c in step)
            sess = session(path, backend, dtype, max_tokens=352, slots=1)
            got = replay(sess, {"a": toks[:n]}, sched)["a"]
            sess.close()
            # (token 7's own query is nothing but rounding noise, which its norm makes as large as any: bf16 holds nine positions in ten,
            # and the asking one, unless it is a neighbour that the second layer's window shows that noise)
            check(got, ref[:n], dtype, f"beacon {beacon} asked at {ask}", share=0.9)
            if dtype == "fp32" or ask - beacon > 3:
                check(got[ask:ask + 1], ref[ask:ask + 1], dtype, f"beacon {beacon} at {ask} itself")
    # the asked position's logits do depend on whether the beacon is inside the window (over the whole context: on its being there)
    for inside, outside, ask in ((0, 299, w - 1), (40, 39 if window else 299, 40 + w - 1)):
        with_it, without = placed(inside, ask)[1][ask][None], placed(outside, ask)[1][ask][None]
        assert rel_err(with_it, without) > 0.15


@pytest.mark.parametrize("backend,dtype", BACKENDS)
def test_previous_token_across_steps(tmp_path, backend, dtype):
    """The bigram row of a portion's first token: the previous token lies in an earlier step, at a block's last place, in a slot and in
    blocks that another request used before, behind a pause in which other requests ran. Nothing but the embedding tells tokens apart
    here, so a wrong row shows at once."""
    cfg = make_config([keyed(2, 1, 8, 1, mlp=dense(16))], vocab=30, width=24, scale=0.05, bigram=(97, 13, 29))
    W = random_weights(cfg, seed=3)
    W["embed"] = (W["embed"].float() * 0.05).to(torch.bfloat16)
    path = save_model(str(tmp_path / "m"), cfg, W)
    reqs = {n: random_tokens(cfg, ln, 60 + i) for i, (n, ln) in enumerate([("a", 70), ("b", 40), ("c", 66), ("d", 35)])}
    sched = [[("a", 32)], [("b", 31), ("a", 1)], [("b", 1)], [("b", 1), ("a", 31)], [("b", 7)], [("c", 2), ("d", 33)], [("d", 1)], [("a", 1), ("c", 30)],
             [("c", 1), ("a", 5)], [("d", 1), ("c", 33)]]
    sess = session(path, backend, dtype, max_tokens=224, slots=3)
    got = replay(sess, reqs, sched)
    sess.close()
    for name, toks in reqs.items():
        check(got[name], oracle_logits(cfg, W, toks), dtype, name)
    other = list(reqs["a"])
    other[31] = (other[31] + 1) % 30
    a, b = oracle_logits(cfg, W, reqs["a"]), oracle_logits(cfg, W, other)
    assert rel_err(a[32:33], b[32:33]) > 0.3           # (the next token's row depends on it)


@pytest.mark.parametrize("backend,dtype", BACKENDS)
def test_long_context(tmp_path, backend, dtype):
    """Hundreds of tokens: whole-context attention over many cache blocks, a window in between, over a prompt, portions and decoding."""
    cfg = make_config([full(4, 2, 16, 16, mlp=dense(32)), keyed(2, 1, 24, 300, mlp=moe(3, 2, 16, shared=16)), full(2, 2, 8, 8, rot=4, mlp=None)],
                      vocab=50, width=32, loop=(0, 2, 2))
    W = random_weights(cfg, seed=9)
    path = save_model(str(tmp_path / "m"), cfg, W)
    toks = random_tokens(cfg, 520, 8)
    sess = session(path, backend, dtype, max_tokens=544, slots=1)
    got = replay(sess, {"a": toks}, [[("a", 330)], [("a", 2)], [("a", 98)]] + [[("a", 1)]] * 90)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, "long", alone(path, backend, dtype, toks), share_of(cfg))


def test_every_mechanism_reaches_the_logits(models):
    """What the tests compare does depend on each piece: changing one moves the plain model's logits by far more than the bounds."""
    cfg, W, _ = models["mixed"]
    toks = random_tokens(cfg, 40, 5)
    ref = oracle_logits(cfg, W, toks)
    for name, change in (("bigram", 0.0), ("loop.in", None), ("l0.mix.g", 0.0), ("l1.mix.q.norm", None), ("l3.mix.k.norm", None), ("l1.norm1b", None),
                         ("l0.norm2b", None), ("l0.mlp.shared.up", 0.0), ("l0.mlp.router", 0.0), ("l4.mlp.gate", None), ("l3.mlp.e1.up", 0.0)):
        W2 = dict(W)
        W2[name] = W[name] * change if change is not None else W[name].flip(0)
        assert rel_err(oracle_logits(cfg, W2, toks), ref) > 0.02, name
    for change in (lambda c: c["embedding"].update(scale=2.0), lambda c: c.update(residual_mult=0.7), lambda c: c["loop"].update(times=1),
                   lambda c: c["loop"].update(start=0), lambda c: c["layers"][1]["mixer"].update(softcap=50.0), lambda c: c["layers"][0]["mixer"]["mask"].update(size=19),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=24), lambda c: c["layers"][3]["mixer"]["rot"].update(base=900.0),
                   lambda c: c["embedding"]["bigram"].update(mul_prev=8), lambda c: c["layers"][4]["mixer"].update(scale=0.5),
                   lambda c: c["layers"][0]["mlp"]["router"].update(top=1)):
        c2 = copy.deepcopy(cfg)
        change(c2)
        assert rel_err(oracle_logits(c2, W, toks), ref) > 0.02
    # the weight on the input of squared-relu experts is not the weight on their output
    import migenex_oracle as O
    h = torch.randn(3, 48, dtype=torch.float64, generator=torch.Generator().manual_seed(1))
    P = O.sub(W, "l0.mlp.")
    assert rel_err((0.5 * O.expert(h, P, "e0.")).numpy(), O.expert(0.5 * h, P, "e0.").numpy()) > 0.2


@pytest.mark.parametrize("stack,buckets", [("mixed", []), ("packed", []), ("mixed", [2]), ("odd_sizes", [1, 2])])
@pytest.mark.parametrize("backend,dtype", BACKENDS)
def test_greedy_generation_through_the_scheduler(models, backend, dtype, stack, buckets):
    """Requests of unequal length through the engine's own entry point: scheduler, continuous batching, chunked prompts,
    sampling (greedy), on the HIP executor with captured decode steps. The tokens are those of the plain model's argmax."""
    from distributed_llm_inference_amd.config import EngineConfig
    from distributed_llm_inference_amd.parallel.launcher import LocalPipeline
    from distributed_llm_inference_amd.runtime.sampler import SamplingParams
    cfg, W, path = models[stack]
    prompts = [random_tokens(cfg, n, 40 + n) for n in (5, 37, 64, 11, 90, 2)]
    new = 24
    ecfg = EngineConfig(model=path, dtype=dtype, pp_size=1, max_batch=4, num_micro_batches=1, max_seq_len=256, prefill_chunk=48,
                        kv_blocks=24, device="cuda" if backend == "hip" else "cpu", backend=backend, seed=0, decode_buckets=buckets)
    pipe = LocalPipeline(ecfg)
    try:
        reqs = [pipe.engine.submit(p, SamplingParams(temperature=0.0, max_new_tokens=new, stop_on_eos=False)) for p in prompts]
        outs = [r.wait(120).output for r in reqs]
        if backend == "hip":
            assert pipe.executors[0].graph_replays > 0, "decode did not go through the captured steps"
    finally:
        pipe.close()
    for p, out in zip(prompts, outs):
        assert len(out) == new
        # teacher-forced: the plain model, fed the engine's own tokens, must agree with every choice (or hold a near tie)
        lg = oracle_logits(cfg, W, p + out)[len(p) - 1:-1]
        for t, row in zip(out, lg):
            best = float(row.max())
            assert row[t] >= best - (1e-3 if dtype == "fp32" else 0.35) * max(1.0, abs(best)), (t, int(row.argmax()))


@pytest.mark.parametrize("backend,dtype,model", [pytest.param("torch", "fp32", "tiny-migenex-test", id="torch"),
                                                 pytest.param("hip", "bf16", "tiny-migenex-gpu-test", id="hip-bf16", marks=pytest.mark.gpu)])
def test_builtin_stack_samples_reproducibly(backend, dtype, model):
    """A built-in Migenex stack (random weights, no checkpoint) through the engine with temperature / top-k / top-p
    sampling: the same seeds give the same tokens on a second pipeline, different seeds do not."""
    from distributed_llm_inference_amd.config import EngineConfig
    from distributed_llm_inference_amd.parallel.launcher import LocalPipeline
    from distributed_llm_inference_amd.runtime.sampler import SamplingParams

    def run(seeds):
        ecfg = EngineConfig(model=model, dtype=dtype, pp_size=1, max_batch=4, num_micro_batches=1, max_seq_len=128, prefill_chunk=32,
                            kv_blocks=16, device="cuda" if backend == "hip" else "cpu", backend=backend, seed=3)
        pipe = LocalPipeline(ecfg)
        try:
            reqs = [pipe.engine.submit(list(range(3, 3 + n)), SamplingParams(temperature=3.0, top_k=40, top_p=0.95, max_new_tokens=12,
                                                                              seed=s, stop_on_eos=False))
                    for n, s in zip((4, 21, 40), seeds)]
            return [r.wait(120).output for r in reqs]
        finally:
            pipe.close()

    a, b, c = run((1, 2, 3)), run((1, 2, 3)), run((4, 5, 6))
    assert all(len(o) == 12 for o in a)
    assert a == b
    assert a != c


def test_config_round_trip_and_export(models, tmp_path):
    """config.json -> spec -> config.json keeps every constant; random weights of a built-in stack, exported under the
    checkpoint's names and loaded again, give the same logits as the plain model on the exported tensors."""
    from distributed_llm_inference_amd.models.partition import make_plans
    from distributed_llm_inference_amd.models.spec import BUILTIN_SPECS, ModelSpec
    from distributed_llm_inference_amd.models.weights import export_migenex_state_dict, random_stage_weights
    for cfg, _, _ in models.values():
        spec = ModelSpec.from_hf_config(cfg)
        again = ModelSpec.from_hf_config(spec.hf_config())
        same = ("layer_specs", "norm_eps", "loop", "loop_input", "bigram", "embed_scale", "residual_mult", "sandwich")
        assert all(getattr(again, k) == getattr(spec, k) for k in same) and spec.residual_mult == cfg["residual_mult"]
        lp = cfg.get("loop") or dict(start=0, stop=0, times=1)
        assert len(spec.layer_runs()) == len(cfg["layers"]) + (lp["stop"] - lp["start"]) * (lp["times"] - 1)
        assert not again.has_recurrent_state            # (the previous token lies in the cache pages: a sequence may change its slot)
    spec = BUILTIN_SPECS["tiny-migenex-test"]
    plan = make_plans(spec, 1)[0]
    w = random_stage_weights(spec, plan, seed=4, dtype=torch.bfloat16)
    sd = export_migenex_state_dict(w)
    path = save_model(str(tmp_path / "m"), spec.hf_config(), sd)
    toks = list(range(5, 45))
    sess = session(path, "torch", "fp32")
    got = replay(sess, {"a": toks}, [[("a", 17)], [("a", 23)]])["a"]
    sess.close()
    check(got, oracle_logits(spec.hf_config(), sd, toks), "fp32", "exported")


@pytest.mark.parametrize("name,cut", [("bigram", lambda t: t[:-1]), ("l2.mix.q", lambda t: t[:-1]), ("loop.in", lambda t: t[:, 1:]), ("head", lambda t: t[1:]),
                                      ("l1.mix.q.norm", lambda t: t[1:]), ("l0.mlp.router", lambda t: t[1:]), ("l0.mix.g", lambda t: t[1:])])
def test_a_checkpoint_that_does_not_fit_its_config_is_refused(models, tmp_path, name, cut):
    cfg, W, _ = models["mixed"]
    bad = dict(W)
    bad[name] = cut(W[name]).contiguous()
    path = save_model(str(tmp_path / "bad"), cfg, bad)
    with pytest.raises(ValueError):
        session(path, "torch", "fp32")


@pytest.mark.parametrize("change", [lambda c: c["layers"][0]["mixer"].update(vdim=8), lambda c: c["layers"][1]["mixer"].update(heads=7),
                                    lambda c: c["loop"].update(stop=6), lambda c: c["loop"].update(times=0), lambda c: c["layers"][0]["mlp"]["router"].update(top=6),
                                    lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), lambda c: c["layers"][1].update(type="delta")])
def test_a_config_that_cannot_be_is_refused(change):
    """Values that are keys of another size, heads that no group divides, a loop beyond the stack, more choices than experts, a rotation
    beyond the head, a mixer that does not exist."""
    from distributed_llm_inference_amd.models.spec import ModelSpec
    cfg = copy.deepcopy(STACKS["mixed"])
    change(cfg)
    with pytest.raises(ValueError):
        ModelSpec.from_hf_config(cfg)


def _random_stack(seed: int):
    """A stack drawn at random: 2 to 5 layers, every size and constant drawn."""
    import random
    rng = random.Random(seed)
    width = rng.choice([24, 40, 64, 96, 128, 136, 200, 256])
    layers = []
    for i in range(rng.randint(2, 5)):
        kind = rng.choice("dmmn")
        mlp = dense(rng.choice([24, 40, 128, 200])) if kind == "d" else None
        if kind == "m":
            E = rng.choice([1, 3, 4, 8, 12])
            mlp = moe(E, rng.randint(1, min(E, 4)), rng.choice([8, 24, 64]), shared=rng.choice([0, 16, 40, 128]))
        G, d = rng.choice([1, 2, 3]), rng.choice([4, 8, 12, 16, 48, 64, 64, 72, 80, 128, 160])
        H, rot, base = G * rng.choice([1, 2, 3, 4, 8]), rng.choice([d, d, d // 2 // 2 * 2, 2, 0]), rng.choice([100.0, 10000.0, 500000.0])
        if rng.random() < 0.5:
            layers.append(full(H, G, d, rng.choice([d, d, 8, 12, 64, 136]), rot=rot, base=base, cap=rng.choice([1.5, 6.0, 30.0]), mlp=mlp))
        else:
            layers.append(keyed(H, G, d, rng.choice([1, 2, 5, 31, 32, 33, 64, 97]), rot=rot, base=base, mlp=mlp))
    a = rng.randrange(len(layers))
    loop = rng.choice([None, (a, rng.randint(a + 1, len(layers)), rng.choice([1, 2, 3]))])
    cfg = make_config(layers, vocab=rng.choice([33, 64, 100, 257]), width=width, loop=loop, mult=rng.choice([0.3, 0.5, 1.0]), scale=rng.choice([1.0, 5.0]),
                      bigram=rng.choice([None, (64, 3, 1), (997, 101, 57)]), eps=rng.choice([1e-5, 1e-6]))
    cuts, left = [], 150
    while left > 0:
        cuts.append(min(left, rng.choice([1, 2, 3, 7, 31, 32, 33, 66])))
        left -= cuts[-1]
    return cfg, cuts


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("seed", [11, 12, 13, 14, 15, 16, 17, 18])
def test_random_stacks(tmp_path, seed, backend, dtype):
    cfg, cuts = _random_stack(seed)
    W = random_weights(cfg, seed=seed)
    path = save_model(str(tmp_path / "m"), cfg, W)
    toks = random_tokens(cfg, sum(cuts) + 15, seed)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", c)] for c in cuts] + [[("a", 1)]] * 15)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, f"seed {seed}", alone(path, backend, dtype, toks), share_of(cfg))


def test_trace_run_executable(models, tmp_path):
    """The executable itself: JSON steps on stdin, `done <step>` lines on stdout, one file of little-endian fp32 logits per
    step in which something is wanted, exit code 0 when the input ends. (CPU: torch executor.)"""
    import json
    import os
    import subprocess
    import sys
    cfg, W, path = models["mixed"]
    a, b = random_tokens(cfg, 40, 71), random_tokens(cfg, 9, 72)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:2], "want": []}, {"id": "a", "tokens": a[33:34], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[34:], "want": [5]}, {"id": "b", "tokens": b[2:], "want": [6]}], "end": ["a", "b"]}]
    exe = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, exe, "--model", path, "--dtype", "float32", "--out", str(out), "--max-tokens", "128",
                        "--backend", "torch", "--device", "cpu"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done ")] == ["done 0", "done 1", "done 2"]
    ra, rb = oracle_logits(cfg, W, a), oracle_logits(cfg, W, b)
    V = cfg["vocab"]
    got = {n: np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, V) for n in (0, 1, 2)}
    check(got[0], ra[[0, 32]], "fp32")
    check(got[1], ra[[33]], "fp32")
    check(got[2], np.stack([ra[39], rb[8]]), "fp32")


def test_generate_command(capsys):
    """The command line's `generate` on a built-in Migenex stack (CPU: torch executor)."""
    import json
    from distributed_llm_inference_amd.serving import cli
    rc = cli.main(["generate", "Hello", "--model", "tiny-migenex-test", "--device", "cpu", "--backend", "torch",
                   "--max-tokens", "5", "--temperature", "0", "--max-seq-len", "128"])
    assert rc == 0
    d = json.loads(capsys.readouterr().out)
    assert d["status"] == "success" and d["tokens_generated"] <= 5 and d["prompt"] == "Hello"
