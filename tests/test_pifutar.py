"""Pifutar through the package (checkpoint reader, executor, cache and state slots, trace replay, scheduler) against the
plain model in `pifutar_oracle`. Every test runs on the torch executor on the CPU; the same tests run on the HIP executor,
in fp32 and in bf16, under the `gpu` marker."""
import numpy as np
import pytest
import torch

from pifutar_util import (SAME, STACKS, TOL, alone, dense, gla, latent, make_config, moe, oracle_logits, random_tokens, random_weights, rel_err,
                          replay, retention, save_model, session)

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


def check(got, ref, dtype, what="", same_as=None, share=1.0, tol=None):
    """`share`: of the positions. (The norm on a head's read-out is a discontinuity where the read-out is nearly zero: at a sequence's
    first token it is (q . k) v, and a q almost orthogonal to its k lets one rounding decide its sign. A stack drawn at random may
    hold such a position.) bf16 against the plain model: nineteen positions in twenty, every one against `same_as`."""
    tol = tol or TOL[dtype]
    e = float(np.quantile(pos_errs(got, ref), share if dtype == "fp32" or len(got) < 20 else min(share, 0.95)))
    assert e < tol, f"{what}: error {e:.3g} over {tol}"
    if same_as is not None:
        e = float(np.quantile(pos_errs(got, same_as.astype(np.float64)), share))
        assert e < SAME[dtype], f"{what}: differs from the whole prompt run alone by {e:.3g}, over {SAME[dtype]}"


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_whole_prompt(models, stack, backend, dtype):
    """Logits, and what goes on from every layer."""
    import pifutar_oracle as O
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
    check(got, ref.numpy(), dtype, stack)


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_prefill_then_token_by_token(models, stack, backend, dtype):
    """A prompt, then decoding one token a step across the windows' edges of every layer and over several cache blocks."""
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, 120, 2)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", 30)]] + [[("a", 1)]] * 90)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, stack, alone(path, backend, dtype, toks))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack", list(STACKS))
def test_first_tokens_alone(models, stack, backend, dtype):
    """A sequence that starts token by token: states from zero, nothing in front of the convolutions."""
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, 12, 3)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", 1)]] * 12)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, stack, alone(path, backend, dtype, toks))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("stack,cuts", [("mixed", [2, 2, 3, 1, 12, 2, 18, 33, 2, 1, 5, 31]), ("odd_sizes", [1, 2, 31, 2, 2, 36, 1, 3, 2, 34, 64, 2]),
                                        ("plain", [2] * 30), ("packed", [2, 31, 2, 1, 97, 3, 130, 2, 33])])
def test_portions(models, stack, cuts, backend, dtype):
    """Prompts cut into portions of changing size, down to two tokens (shorter than the convolutions' reach), in the middle of
    cache blocks, windows and the recurrences' chunks."""
    cfg, W, path = models[stack]
    toks = random_tokens(cfg, sum(cuts), 4)
    sess = session(path, backend, dtype)
    got = replay(sess, {"a": toks}, [[("a", c)] for c in cuts])["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, stack, alone(path, backend, dtype, toks))


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
        check(got[name], oracle_logits(cfg, W, toks), dtype, f"{stack}/{name}", alone(path, backend, dtype, toks))


@pytest.mark.parametrize("backend,dtype", BACKENDS)
def test_slot_taken_over_starts_clean(models, backend, dtype):
    """One slot, one request after another: the second must not see the first one's states, convolution inputs or cache rows."""
    cfg, W, path = models["mixed"]
    a, b = random_tokens(cfg, 50, 31), random_tokens(cfg, 20, 32)
    sess = session(path, backend, dtype, max_tokens=64, slots=1)
    got = replay(sess, {"a": a, "b": b}, [[("a", 50)], [("b", 1)], [("b", 2)], [("b", 17)]])
    sess.close()
    check(got["b"], oracle_logits(cfg, W, b), dtype, "second", alone(path, backend, dtype, b))
    check(got["a"], oracle_logits(cfg, W, a), dtype, "first", alone(path, backend, dtype, a))


def _beacon_model(windows):
    """Latent layers of one rank entry each whose single key stands out: token 7's latent is large along an entry that token 9 asks
    for. The second layer reads the first one's latents through a window of its own."""
    cfg = make_config([latent(2, 8, 4, 12, 16, window=windows[0], scale=1.0), latent(3, 8, 4, 8, 16, window=windows[1], kv_from=0, scale=1.0)],
                      vocab=40, width=32, taps=1)
    W = random_weights(cfg, seed=5)
    e7, e9 = W["embed"][7].float(), W["embed"][9].float()
    # token 7 and 9 orthogonal to each other and of equal length, the others free of both directions
    e9 = e9 - e7 * (e9 @ e7) / (e7 @ e7)
    e9 = e9 * e7.norm() / e9.norm()
    E = W["embed"].float()
    for t in range(40):
        for u in (e7, e9):
            E[t] = E[t] - u * (E[t] @ u) / (u @ u)
    E[7], E[9] = e7, e9
    W["embed"] = E.to(torch.bfloat16)
    for i in (0, 1):
        W[f"l{i}.norm1"] = torch.zeros(32, dtype=torch.bfloat16)
        W[f"l{i}.canon1"] = torch.zeros(32, 1, dtype=torch.bfloat16)
        W[f"l{i}.dwa"] = torch.tensor([1.0] + [0.0] * i + [0.5], dtype=torch.bfloat16)      # (the embedding stays the larger part of what is read)
        q = torch.zeros_like(W[f"l{i}.mix.q"].float())
        d, dr = 8, 4
        q[::d + dr] = 0.5 * e9                    # every head's first unrotated query entry asks
        W[f"l{i}.mix.q"] = q.to(torch.bfloat16)
        uk = torch.zeros_like(W[f"l{i}.mix.uk"].float())
        uk[::d, 0] = 2.0
        W[f"l{i}.mix.uk"] = uk.to(torch.bfloat16)
        W[f"l{i}.mix.o"] = (W[f"l{i}.mix.o"].float() * 3.0).to(torch.bfloat16)
    W["l0.mix.dkv"][0] = (0.5 * e7).to(torch.bfloat16)
    W["l0.mix.dkv.norm"] = torch.ones(16, dtype=torch.bfloat16)
    return cfg, W


@pytest.mark.parametrize("backend,dtype", BACKENDS)
@pytest.mark.parametrize("layer,windows", [(0, (130, 1)), (1, (1, 130))])
def test_window_edges_and_far_keys(tmp_path, backend, dtype, layer, windows):
    """A key that stands out at the window's last place, one position outside, right behind the asking token and across cache
    blocks; in a prompt, in portions cut around the asking token, and in decoding; for a layer's own latents and for latents read
    from another layer. A window that is one token off moves the logits by far more than the tolerance."""
    cfg, W = _beacon_model(windows)
    path = save_model(str(tmp_path / "m"), cfg, W)
    base = [t for t in random_tokens(cfg, 500, 6) if t not in (7, 9)][:300]

    def placed(beacon, ask):
        toks = list(base)
        toks[beacon], toks[ask] = 7, 9
        return toks, oracle_logits(cfg, W, toks)

    for beacon, ask in [(0, 129), (0, 130), (130, 259), (129, 259), (130, 131), (31, 160), (32, 162), (200, 250)]:
        toks, ref = placed(beacon, ask)
        for sched in ([[("a", 300)]], [[("a", ask - 1)], [("a", 2)], [("a", 300 - ask - 1)]], [[("a", ask)]] + [[("a", 1)]] * 3):
            n = sum(c for step in sched for _, c in step)
            sess = session(path, backend, dtype, max_tokens=352, slots=1)
            got = replay(sess, {"a": toks[:n]}, sched)["a"]
            sess.close()
            check(got, ref[:n], dtype, f"beacon {beacon} asked at {ask}")
    # the asked position's logits do depend on whether the beacon is inside the window
    for inside, outside, ask in ((0, 1, 129), (130, 129, 259)):
        with_it, without = placed(inside, ask)[1][ask][None], placed(outside if outside < inside else 299, ask)[1][ask][None]
        assert rel_err(with_it, without) > 0.15


@pytest.mark.parametrize("backend,dtype", BACKENDS)
def test_long_memories(tmp_path, backend, dtype):
    """Decays close to one: hundreds of tokens stay in the states over a prompt of many chunks, portions and decoding."""
    cfg = make_config([retention(3, 16, 16, decay=[1.0, 0.9995, 0.99], mlp=dense(32)), gla(2, 24, 16, tau=64.0, rank=4, mlp=moe(3, 2, 16, shared=16)),
                       latent(2, 8, 8, 16, 24, window=300)], vocab=50, width=32, taps=2)
    W = random_weights(cfg, seed=9)
    W["l1.mix.a2.b"] = W["l1.mix.a2.b"] + 3.0
    path = save_model(str(tmp_path / "m"), cfg, W)
    toks = random_tokens(cfg, 520, 8)
    sess = session(path, backend, dtype, max_tokens=544, slots=1)
    got = replay(sess, {"a": toks}, [[("a", 330)], [("a", 2)], [("a", 98)]] + [[("a", 1)]] * 90)["a"]
    sess.close()
    check(got, oracle_logits(cfg, W, toks), dtype, "long", alone(path, backend, dtype, toks))


def test_every_mechanism_reaches_the_logits(models):
    """What the tests compare does depend on each piece: leaving one out moves the plain model's logits by far more than the bounds."""
    cfg, W, _ = models["mixed"]
    toks = random_tokens(cfg, 40, 5)
    ref = oracle_logits(cfg, W, toks)
    for name, change in (("l0.canon1", 0.0), ("l3.canon1", 0.0), ("l2.canon2", 0.0), ("l4.dwa", None), ("l2.mix.a2", 0.0), ("l2.mix.norm", 0.0),
                         ("l1.mlp.act", None), ("l0.mlp.shared.sg", 0.0), ("l1.mix.dkv.norm", None), ("l0.mlp.table", "shift")):
        W2 = dict(W)
        t = W[name]
        W2[name] = (t + 1) % 5 if change == "shift" else t * change if change is not None else t.flip(0)
        assert rel_err(oracle_logits(cfg, W2, toks), ref) > 0.02, name


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


@pytest.mark.parametrize("backend,dtype,model", [pytest.param("torch", "fp32", "tiny-pifutar-test", id="torch"),
                                                 pytest.param("hip", "bf16", "tiny-pifutar-gpu-test", id="hip-bf16", marks=pytest.mark.gpu)])
def test_builtin_stack_samples_reproducibly(backend, dtype, model):
    """A built-in Pifutar stack (random weights, no checkpoint) through the engine with temperature / top-k / top-p
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
    from distributed_llm_inference_amd.models.weights import export_pifutar_state_dict, random_stage_weights
    for cfg, _, _ in models.values():
        spec = ModelSpec.from_hf_config(cfg)
        again = ModelSpec.from_hf_config(spec.hf_config())
        assert again.layer_specs == spec.layer_specs and again.norm_eps == spec.norm_eps and again.input_conv == spec.input_conv == cfg["canon"]["taps"]
        assert again.has_recurrent_state
    spec = BUILTIN_SPECS["tiny-pifutar-test"]
    plan = make_plans(spec, 1)[0]
    w = random_stage_weights(spec, plan, seed=4, dtype=torch.bfloat16)
    sd = export_pifutar_state_dict(w)
    path = save_model(str(tmp_path / "m"), spec.hf_config(), sd)
    toks = list(range(5, 45))
    sess = session(path, "torch", "fp32")
    got = replay(sess, {"a": toks}, [[("a", 17)], [("a", 23)]])["a"]
    sess.close()
    check(got, oracle_logits(spec.hf_config(), sd, toks), "fp32", "exported")


@pytest.mark.parametrize("name,cut", [("l0.mlp.table", lambda t: t[:, :1]), ("l0.mlp.table", lambda t: t + 4), ("l2.mix.q", lambda t: t[:-1]),
                                      ("l3.dwa", lambda t: t[:-1]), ("l1.canon1", lambda t: t[:, 1:])])
def test_a_checkpoint_that_does_not_fit_its_config_is_refused(models, tmp_path, name, cut):
    cfg, W, _ = models["mixed"]
    bad = dict(W)
    bad[name] = cut(W[name]).contiguous()
    path = save_model(str(tmp_path / "bad"), cfg, bad)
    with pytest.raises(ValueError):
        session(path, "torch", "fp32")


@pytest.mark.parametrize("layers", [[gla(2, 8, 8), latent(2, 8, 4, 8, 16, kv_from=0)], [latent(2, 8, 4, 8, 16), latent(2, 8, 4, 8, 20, kv_from=0)],
                                    [latent(2, 8, 4, 8, 16), latent(2, 8, 4, 8, 16, kv_from=1)], [retention(3, 8, 8, decay=[0.5, 0.5])]])
def test_a_config_that_cannot_be_is_refused(layers):
    """Latents of a layer that keeps none, of another size, of the layer itself; as many decays as heads."""
    from distributed_llm_inference_amd.models.spec import ModelSpec
    with pytest.raises(ValueError):
        ModelSpec.from_hf_config(make_config(layers, vocab=20, width=16))


def _random_stack(seed: int):
    """A stack drawn at random: 2 to 6 layers, every size and constant drawn."""
    import random
    rng = random.Random(seed)
    width = rng.choice([24, 40, 64, 96, 128, 136, 200, 256])
    layers, sources = [], []
    for i in range(rng.randint(2, 6)):
        kind = rng.choice("dmmn")
        mlp = dense(rng.choice([24, 40, 128, 200])) if kind == "d" else None
        if kind == "m":
            E = rng.choice([1, 3, 4, 8, 12])
            mlp = moe(E, rng.randint(1, min(E, 4)), rng.choice([8, 24, 64]), limit=rng.choice([0.5, 1.0, 7.0]), shared=rng.choice([0, 16, 40, 128]),
                      shared_limit=rng.choice([0.6, 5.0]))
        heads, t = rng.choice([1, 2, 3, 4, 6, 8, 20]), rng.choice("grls")
        if t == "g":
            layers.append(gla(heads, rng.choice([4, 12, 16, 48, 64, 80]), rng.choice([8, 12, 32, 64, 136]), tau=rng.choice([1.0, 4.0, 16.0]), rank=rng.choice([1, 4, 16]), mlp=mlp))
        elif t == "r":
            layers.append(retention(heads, rng.choice([4, 12, 16, 48, 64, 80]), rng.choice([8, 12, 32, 64, 136]),
                                    decay=[rng.choice([0.3, 0.9, 0.99, 0.999, 1.0]) for _ in range(heads)], mlp=mlp))
        else:
            src = rng.choice(sources) if t == "s" and sources else None
            R, dr, base = src[1:] if src else (rng.choice([8, 16, 20, 64, 128, 200]), rng.choice([2, 4, 8, 16, 32]), rng.choice([100.0, 10000.0, 500000.0]))
            if src is None:
                sources.append((i, R, dr, base))
            layers.append(latent(heads, rng.choice([4, 8, 12, 32, 48]), dr, rng.choice([8, 12, 32, 64]), R, window=rng.choice([0, 1, 2, 5, 31, 32, 33, 64, 97]), base=base,
                                 kv_from=src[0] if src else None, mlp=mlp))
    cfg = make_config(layers, vocab=rng.choice([33, 64, 100, 257]), width=width, taps=rng.choice([1, 2, 3, 4, 6]), eps=rng.choice([1e-5, 1e-6]))
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
    check(got, oracle_logits(cfg, W, toks), dtype, f"seed {seed}", alone(path, backend, dtype, toks), share=0.9)


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
    """The command line's `generate` on a built-in Pifutar stack (CPU: torch executor)."""
    import json
    from distributed_llm_inference_amd.serving import cli
    rc = cli.main(["generate", "Hello", "--model", "tiny-pifutar-test", "--device", "cpu", "--backend", "torch",
                   "--max-tokens", "5", "--temperature", "0", "--max-seq-len", "128"])
    assert rc == 0
    d = json.loads(capsys.readouterr().out)
    assert d["status"] == "success" and d["tokens_generated"] <= 5 and d["prompt"] == "Hello"
