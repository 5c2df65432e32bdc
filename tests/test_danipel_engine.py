"""The Danipel family inside the engine (registry, loader, scheduler, paged latent cache, kernels)
against the plain oracle of ``danipel_oracle``: every mechanism alone (one-layer models), whole
prompts and the summed streams after every layer, token-by-token decoding, portions down to two
tokens, mixed batches against each request alone, blocks that are used again, a key that stands
out at the first token / at block borders / next to the query / hundreds of positions back (in
prompts and while decoding), long decoding, sizes that are 1 or equal, configurations drawn at
random, prefixes found in the cache, greedy generation through ``LLMEngine.generate``, and the
replay entry point.  Every test runs on the CPU (fp32); the ``gpu`` variants run the HIP kernels
in float32 and bfloat16."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import danipel_fixtures as fx
import danipel_oracle as oracle

from minivllm_amd.engine.llm_engine import LLMEngine
from minivllm_amd.models.registry import config_from_path
from minivllm_amd.sampling_parameters import SamplingParams

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CASES = [pytest.param("cpu", "float32", id="cpu-fp32"),
         pytest.param("cuda", "float32", id="gpu-fp32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu)]


def make_engine(tmp_path, c, w, device, dtype, blocks=24, block_size=8, seqs=3, score=True, **kw):
    folder = fx.save_checkpoint(str(tmp_path / "ckpt"), c, w)
    mc = config_from_path(folder)
    assert type(mc).__name__ == "DanipelConfig"
    cfg = dict(model=mc, checkpoint_path=folder, dtype=dtype, device=device,
               block_size=block_size, max_cached_blocks=blocks, max_num_sequences=seqs,
               max_model_length=blocks * block_size,
               max_num_batched_tokens=blocks * block_size, eos=-1, score_only=score,
               graph_batch_sizes=[1, 2, seqs], tuned_gemms=False)
    cfg.update(kw)
    return LLMEngine(cfg)


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


class Expected:
    def __init__(self, c, w, toks):
        self.logits, self.trace = oracle.forward(c, w, toks)


def close(got, want, dtype):
    """Error of a logit row: spread of the difference over the vocabulary relative to the spread
    of the logits themselves.  In bfloat16 a router whose two best logits nearly tie may choose
    the other expert, which moves that row: a twentieth of the rows may lie beyond the limit."""
    d = got.double() - want.logits
    d = d - d.mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / want.logits.std(-1)
    if dtype == "float32":
        assert float(e.max()) < 2e-4, f"logits differ: {float(e.max()):.3g} at {int(e.argmax())}"
    else:
        assert float(e.median()) < 0.06, f"typical row differs: {float(e.median()):.3g}"
        assert float((e > 0.3).float().mean()) <= 0.05, f"{int((e > 0.3).sum())} of {len(e)} rows differ"


def run_schedule(eng, reqs, schedule):
    """``schedule``: list of steps, each a list of (name, count).  Returns name -> [len, V]."""
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    for step in schedule:
        entries, end = [], []
        for name, n in step:
            lo = at[name]
            entries.append({"id": name, "tokens": reqs[name][lo:lo + n], "want": list(range(n))})
            at[name] = lo + n
            if at[name] == len(reqs[name]):
                end.append(name)
        out = eng.score_step(entries, end)
        for name, _ in step:
            got[name].append(out[name])
    return {k: torch.cat(v) for k, v in got.items() if v}


ALONE = {
    "latent-sink-yarn": [(fx.latent(1, scaling=fx.YARN), None)],
    "latent-sink": [(fx.latent(1), None)],
    "latent-low-rank": [(fx.latent(2), None)],
    "latent-low-rank-yarn": [(fx.latent(2, scaling=fx.YARN), None)],
    "one-head": [(fx.latent(1, heads=1, dim=7, rot_dim=2, vdim=3, kv_rank=9), None)],
    "latent-serving-sizes": [(fx.latent(1, heads=16, dim=64, rot_dim=64, vdim=64, kv_rank=128, scale=0.09), None)],
    "latent-wide": [(fx.latent(2, heads=8, dim=32, rot_dim=64, vdim=32, kv_rank=256, q_rank=96, scale=0.1), None)],
    "dense": [(fx.latent(2), fx.dense())],
    "experts": [(fx.latent(2), fx.moe())],
    "experts-no-shared": [(fx.latent(1), fx.moe(experts=6, identity=1, top=3, ff=8, shared_ff=0))],
    "experts-mostly-identity": [(fx.latent(1), fx.moe(experts=2, identity=6, top=5, ff=8))],
}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", list(ALONE))
def test_each_mechanism_alone(tmp_path, device, dtype, kind):
    """One-layer models: whole prompt, then the same tokens as a prompt portion + single tokens."""
    c = fx.config(ALONE[kind], width=32, vocab=53, streams=2)
    w = fx.weights(c, 40)
    toks = tokens(33, c["vocab"], 41)
    eng = make_engine(tmp_path, c, w, device, dtype)
    seen = []
    eng.model_runner.model.model.layer_hook = lambda i, x: seen.append(x.detach().float().cpu().clone())
    want = Expected(c, w, toks)
    close(run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"], want, dtype)
    lim = 1e-4 if dtype == "float32" else 0.1
    n = len(toks)
    if dtype == "float32" or "experts" not in kind:
        assert float((seen[0][:n].double() - want.trace[0]).abs().max()) < lim * float(want.trace[0].abs().max())
    eng.model_runner.model.model.layer_hook = None
    close(run_schedule(eng, {"b": toks}, [[("b", 5)], [("b", 17)]] + [[("b", 1)]] * 11)["b"], want, dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_whole_prompt_and_every_layer(tmp_path, device, dtype):
    c = fx.default_config()
    w = fx.weights(c, 103)
    toks = tokens(37, c["vocab"], 2)
    eng = make_engine(tmp_path, c, w, device, dtype)
    seen = []
    eng.model_runner.model.model.layer_hook = lambda i, x: seen.append(x.detach().float().cpu().clone())
    got = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    want = Expected(c, w, toks)
    close(got, want, dtype)
    assert len(seen) == len(c["layers"])
    if dtype == "float32":
        for x, ref in zip(seen, want.trace):
            assert float((x[:len(toks)].double() - ref).abs().max()) < 1e-4 * float(ref.abs().max())
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_token_by_token_equals_prefill(tmp_path, device, dtype):
    c = fx.default_config()
    w = fx.weights(c, 3)
    toks = tokens(29, c["vocab"], 4)
    eng = make_engine(tmp_path, c, w, device, dtype)
    want = Expected(c, w, toks)
    close(run_schedule(eng, {"a": toks}, [[("a", 1)] for _ in toks])["a"], want, dtype)   # first tokens, then decode
    close(run_schedule(eng, {"b": toks}, [[("b", 20)]] + [[("b", 1)]] * 9)["b"], want, dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("cuts", [[2, 2, 3, 1, 9, 8, 2, 16, 2, 5], [7, 43], [1, 2, 47], [25, 25]])
def test_portions_cut_anywhere(tmp_path, device, dtype, cuts):
    c = fx.default_config()
    w = fx.weights(c, 5)
    toks = tokens(sum(cuts), c["vocab"], 6)
    eng = make_engine(tmp_path, c, w, device, dtype)
    got = run_schedule(eng, {"a": toks}, [[("a", n)] for n in cuts])["a"]
    close(got, Expected(c, w, toks), dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_mixed_batches_equal_each_request_alone(tmp_path, device, dtype):
    c = fx.default_config()
    w = fx.weights(c, 7)
    reqs = {"a": tokens(41, c["vocab"], 8), "b": tokens(5, c["vocab"], 9), "c": tokens(23, c["vocab"], 10),
            "d": tokens(1, c["vocab"], 11), "e": tokens(18, c["vocab"], 12)}
    sched = [[("a", 9), ("b", 2)],
             [("a", 1), ("b", 1), ("c", 17)],              # a one-token portion next to a prompt
             [("b", 1), ("c", 1)],                         # decode step of two; a sits out
             [("a", 20), ("b", 1), ("c", 1)],              # b ends: its blocks return
             [("a", 1), ("c", 1), ("d", 1)],               # d's first token alone
             [("e", 3), ("a", 1), ("c", 1)],
             [("e", 15), ("a", 9), ("c", 2)]]
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=14, seqs=3)
    got = run_schedule(eng, reqs, sched)
    for k, toks in reqs.items():
        close(got[k], Expected(c, w, toks), dtype)
    bm = eng.scheduler.block_manager
    assert bm.num_free_blocks == bm.num_blocks
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_pool_used_again(tmp_path, device, dtype):
    """A KV pool of just over one request: every later request runs on blocks that an earlier one
    has left dirty."""
    c = fx.default_config()
    w = fx.weights(c, 13)
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=9, seqs=2)
    for i, n in enumerate([60, 33, 64, 9, 2]):
        toks = tokens(n, c["vocab"], 20 + i)
        cut = max(1, n // 3)
        got = run_schedule(eng, {"r": toks}, [[("r", cut)], [("r", n - cut)]] if n > 1 else [[("r", 1)]])["r"]
        close(got, Expected(c, w, toks), dtype)
    eng.exit()


def _swap(t):
    h = t.shape[-1] // 2
    return torch.cat([t[..., h:], t[..., :h]], -1).contiguous()


def _standout_model(kind):
    """One latent layer made so that ONE key stands out for the last query: token 38's embedding is
    token 39's with its halves swapped, and head 1's unrotated query path is the latent's own with
    its input columns swapped the same way (the norm treats all columns alike), so q_1(token 39)
    is a multiple of the latent of token 38 - wherever that sits - while head 1's unrotated key IS
    the latent.  A small rotated part, a deep sink."""
    W, R = 32, 16
    c = fx.config([(fx.latent(kind, heads=2, dim=R, rot_dim=4, vdim=R, kv_rank=R, q_rank=R, scale=0.5), None)],
                  width=W, vocab=40, streams=2)
    w = fx.weights(c, 50)
    p = "l0.mix."
    w["l0.norm1"], w["l0.norm1.b"] = torch.ones_like(w["l0.norm1"]), torch.zeros_like(w["l0.norm1.b"])
    latent = w[p + "dkv"][:R]
    w[p + "dkv.norm"] = torch.ones_like(w[p + "dkv.norm"])
    uk = w[p + "uk"].clone()
    uk[R:2 * R] = torch.eye(R)
    w[p + "uk"] = uk
    q1 = slice(R + 4, 2 * R + 4)                                   # head 1's unrotated rows of q
    if kind == 1:
        q = w[p + "q"].clone()
        q[q1] = 3.0 * _swap(latent)
        w[p + "q"] = q
        w[p + "sink"] = torch.full_like(w[p + "sink"], -4.0)
    else:
        w[p + "dq"] = _swap(latent)
        w[p + "dq.norm"] = torch.ones_like(w[p + "dq.norm"])
        uq = w[p + "uq"].clone()
        uq[q1] = 2.0 * torch.eye(R)
        w[p + "uq"] = uq
    e = w["embed"].clone()
    e[38] = _swap(e[39])
    w["embed"] = e
    return c, {k: v.to(torch.bfloat16) for k, v in w.items()}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decoded", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("kind", [1, 2])
@pytest.mark.parametrize("n", [41, 330], ids=["short", "far"])
def test_a_key_that_stands_out(tmp_path, device, dtype, decoded, kind, n):
    """Token 38 sits at one key position, token 39 at the last one, which asks for it: at the first
    token, on both sides of a page border, on both sides of the kernels' runs of keys (32, 64, 256),
    right before the query.  The oracle's logits with and without the key differ widely, so a key
    that is missed or misplaced cannot pass."""
    bs = 8
    c, w = _standout_model(kind)
    q = n - 1
    places = [0, 1, bs - 1, bs, 31, 32, q - 1, q - 6] + ([63, 64, 127, 128, 255, 256] if n > 300 else [])
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=n // bs + 4, block_size=bs, seqs=2)
    base = [1 + (t * 7) % 37 for t in range(n)]                    # ids 1 .. 37
    base[q] = 39
    without = oracle.forward(c, w, base)[0][q]
    for where in places:
        toks = list(base)
        toks[where] = 38
        sched = [[("a", n)]] if not decoded else [[("a", n - 6)]] + [[("a", 1)]] * 6
        got = run_schedule(eng, {"a": toks}, sched)["a"]
        want = Expected(c, w, toks)
        close(got, want, dtype)
        assert float((want.logits[q] - without).std()) > 0.2 * float(without.std()), "the key does not stand out"
        if dtype == "bfloat16":
            assert float((got[q].double() - want.logits[q]).std()) < 0.3 * float((want.logits[q] - without).std())
    eng.exit()


def test_sink_scaling_and_mix_show(tmp_path):
    """The oracle with the sink taken out, without YaRN, with the mix transposed or with the
    correction added to the weights' choice left out gives other logits than the engine: no
    mechanism hides behind the random weights."""
    c = fx.config([(fx.latent(1, scaling=fx.YARN), fx.moe())], width=32, vocab=53)
    w = fx.weights(c, 44)
    toks = tokens(25, c["vocab"], 45)
    eng = make_engine(tmp_path, c, w, "cpu", "float32")
    got = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    close(got, Expected(c, w, toks), "float32")
    c2 = json.loads(json.dumps(c))
    del c2["layers"][0]["mixer"]["rot"]["scaling"]
    others = [(c, dict(w, **{"l0.mix.sink": torch.full_like(w["l0.mix.sink"], -60.0)})), (c2, w),
              (c, dict(w, **{"l0.hc1.mix": w["l0.hc1.mix"].T.contiguous()})),
              (c, dict(w, **{"l0.mlp.correction": torch.zeros_like(w["l0.mlp.correction"])}))]
    for cc, ww in others:
        far = oracle.forward(cc, ww, toks)[0]
        assert float((got.double() - far).std()) > 0.02 * float(far.std())
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_decoding_over_many_blocks(tmp_path, device, dtype):
    """150 single tokens behind a prompt of three: many page borders, YaRN past its original length."""
    c = fx.config([(fx.latent(1, heads=2, dim=8, rot_dim=6, vdim=4, kv_rank=12, scaling=fx.YARN),
                    fx.moe(experts=3, top=2, ff=8, shared_ff=8)),
                   (fx.latent(2, heads=2, dim=8, rot_dim=8, vdim=8, kv_rank=8), fx.dense(16))], width=24, vocab=61)
    w = fx.weights(c, 14)
    toks = tokens(150, c["vocab"], 15)
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=40, block_size=4)
    got = run_schedule(eng, {"a": toks}, [[("a", 3)]] + [[("a", 1)]] * 147)["a"]
    close(got, Expected(c, w, toks), dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_sizes_that_happen_to_be_one_or_equal(tmp_path, device, dtype):
    """One head, a latent of one number, one stream, one expert, only identity experts chosen, top =
    all, no feed-forward anywhere, scales of one, every size the same, a scaling factor of one."""
    for layers, extra in (
            ([(fx.latent(1, heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, scale=1.0), fx.moe(experts=1, identity=1, top=2, ff=8, shared_ff=8))],
             dict(streams=1, residual_mult=1.0, embed_scale=1.0)),
            ([(fx.latent(2, heads=4, dim=16, rot_dim=16, vdim=16, kv_rank=16, q_rank=16, scale=1.0), fx.dense(16)),
              (fx.latent(1, heads=4, dim=16, rot_dim=16, vdim=16, kv_rank=16,
                         scaling={"factor": 1.0, "original": 16, "fast": 1.0, "slow": 1.0}), None)], dict(streams=4)),
            ([(fx.latent(1, heads=5, dim=6, rot_dim=6, vdim=6, kv_rank=30), fx.moe(experts=2, identity=0, top=1, scale=1.0)),
              (fx.latent(2, heads=3, dim=4, rot_dim=10, vdim=2, kv_rank=6, q_rank=1), None)], dict(streams=8))):
        c = fx.config(layers, width=16, vocab=50, **extra)
        w = fx.weights(c, 16)
        toks = tokens(21, c["vocab"], 17)
        eng = make_engine(tmp_path, c, w, device, dtype)
        got = run_schedule(eng, {"a": toks}, [[("a", 2)], [("a", 12)]] + [[("a", 1)]] * 7)["a"]
        close(got, Expected(c, w, toks), dtype)
        eng.exit()


def _random_config(seed):
    """A configuration drawn from a seed: widths, streams, head counts and sizes (also odd ones and
    latents above 256), layer order, rotations, experts and constants."""
    g = torch.Generator().manual_seed(seed)

    def pick(*xs):
        return xs[int(torch.randint(0, len(xs), (1,), generator=g))]
    layers = []
    for _ in range(pick(2, 3, 4)):
        m = fx.latent(pick(1, 2), heads=pick(1, 3, 6, 12, 17), dim=pick(8, 24, 32, 64), rot_dim=pick(4, 16, 32),
                      vdim=pick(8, 20, 64), kv_rank=pick(24, 96, 128, 288), q_rank=pick(16, 50),
                      scale=pick(0.1, 0.2), base=pick(10.0, 10000.0, 1e6),
                      scaling=pick(None, fx.YARN, {"factor": 2.0, "original": 1000, "fast": 32.0, "slow": 1.0}))
        ne, ni = pick(2, 4, 7), pick(0, 1, 3)
        layers.append((m, pick(None, fx.dense(pick(8, 40, 96)),
                               fx.moe(experts=ne, identity=ni, top=pick(1, 2, ne), ff=pick(8, 20, 48),
                                      limit=pick(0.5, 2.0, 7.0), scale=pick(1.0, 2.5), shared_ff=pick(0, 8, 40),
                                      shared_limit=pick(0.5, 3.0)))))
    return fx.config(layers, width=pick(24, 50, 96, 160), vocab=pick(50, 131), eps=pick(1e-6, 1e-5),
                     streams=pick(1, 2, 3, 4), residual_mult=pick(0.4, 1.0), embed_scale=pick(1.0, 5.0, 12.0))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("seed", list(range(8)))
def test_configurations_drawn_at_random(tmp_path, device, dtype, seed):
    c = _random_config(seed)
    w = fx.weights(c, 70 + seed, qk_gain=1.0)
    toks = tokens(45, c["vocab"], 80 + seed)
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=16, block_size=8)
    want = Expected(c, w, toks)
    close(run_schedule(eng, {"a": toks}, [[("a", 45)]])["a"], want, dtype)
    close(run_schedule(eng, {"b": toks}, [[("b", 7)], [("b", 2)], [("b", 26)]] + [[("b", 1)]] * 10)["b"], want, dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_equal_prefixes_share_blocks(tmp_path, device, dtype):
    """Live requests with a common prefix, in the same step and in later ones, scored in other
    portions: what is shared in the cache is the same for all of them."""
    c = fx.default_config()
    w = fx.weights(c, 90)
    head = tokens(20, c["vocab"], 91)
    reqs = {"a": head + tokens(6, c["vocab"], 92), "b": head + tokens(9, c["vocab"], 93), "c": list(head) + [3]}
    eng = make_engine(tmp_path, c, w, device, dtype)
    got = run_schedule(eng, reqs, [[("a", 20), ("b", 17)], [("b", 4), ("c", 19), ("a", 1)], [("a", 2), ("c", 1)],
                                   [("c", 1), ("b", 2), ("a", 1)], [("b", 6), ("a", 2)]])
    for k, toks in reqs.items():
        close(got[k], Expected(c, w, toks), dtype)
    assert eng.scheduler.block_manager.num_free_blocks == eng.scheduler.block_manager.num_blocks
    eng.exit()


def _follow(c, w, prompt, gen, dtype):
    """Greedy tokens against the oracle (recomputed from scratch per token: it keeps no state)."""
    toks = list(prompt)
    for t in gen:
        lg = oracle.forward(c, w, toks)[0][-1]
        top2 = lg.topk(2).values
        if dtype == "bfloat16" and float(top2[0] - top2[1]) < 0.15:
            break                          # a near tie: 16-bit rounding may pick either
        if dtype == "bfloat16" and int(lg.argmax()) != t:
            break                          # (a router's near tie upstream; the fp32 cases are exact)
        assert int(lg.argmax()) == t
        toks.append(t)


@pytest.mark.parametrize("device,dtype", CASES)
def test_greedy_generation_through_the_scheduler(tmp_path, device, dtype):
    c = fx.default_config()
    w = fx.weights(c, 18)
    prompts = [tokens(n, c["vocab"], 30 + n) for n in (11, 3, 26, 1)]
    eng = make_engine(tmp_path, c, w, device, dtype, score=False, seqs=3, blocks=30,
                      max_num_batched_tokens=32)
    out = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True))
    for p, gen in zip(prompts, out["token_ids"]):
        assert len(gen) == 8
        _follow(c, w, p, gen, dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_generation_reuses_a_cached_prefix(tmp_path, device, dtype):
    c = fx.default_config()
    w = fx.weights(c, 24)
    head = tokens(24, c["vocab"], 25)
    eng = make_engine(tmp_path, c, w, device, dtype, score=False, seqs=2, blocks=30)
    for n in (5, 7):
        prompt = head + tokens(n, c["vocab"], 26 + n)
        out = eng.generate([prompt], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
        _follow(c, w, prompt, out["token_ids"][0], dtype)
    assert eng.scheduler.block_manager.num_prefix_hits >= 3
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES[:2])
def test_generation_survives_preemption_and_mixed_steps(tmp_path, device, dtype):
    c = fx.default_config()
    w = fx.weights(c, 19)
    prompts = [tokens(n, c["vocab"], 60 + n) for n in (21, 17, 9, 30)]
    eng = make_engine(tmp_path, c, w, device, dtype, score=False, seqs=3, blocks=11, block_size=8,
                      max_num_batched_tokens=24, enable_mixed_batches=True)
    out = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=14, ignore_eos=True))
    assert eng.scheduler.num_preemptions > 0 and eng.scheduler.num_mixed_steps > 0
    for p, gen in zip(prompts, out["token_ids"]):
        _follow(c, w, p, gen, dtype)
    eng.exit()


def test_replay_entry_point_writes_the_oracles_logits(tmp_path):
    c = fx.default_config()
    w = fx.weights(c, 21)
    folder = fx.save_checkpoint(str(tmp_path / "m"), c, w)
    a, b = tokens(70, c["vocab"], 22), tokens(9, c["vocab"], 23)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [0, 39]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[40:69], "want": []},
                                     {"id": "b", "tokens": b[:8], "want": [7]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]},
                                     {"id": "a", "tokens": a[69:], "want": [0]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder,
                        "--dtype", "float32", "--out", str(out), "--max-tokens", "192",
                        "--block-size", "16", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = oracle.forward(c, w, a)[0].float().numpy(), oracle.forward(c, w, b)[0].float().numpy()
    V = c["vocab"]
    got = {n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, V) for n in range(3)}
    np.testing.assert_allclose(got[0], la[[0, 39]], rtol=2e-4, atol=2e-4)
    np.testing.assert_allclose(got[1], lb[[7]], rtol=2e-4, atol=2e-4)
    np.testing.assert_allclose(got[2], np.stack([lb[8], la[69]]), rtol=2e-4, atol=2e-4)


def test_checkpoint_errors_name_the_tensor(tmp_path):
    c = fx.config([(fx.latent(1), fx.moe()), (fx.latent(2), fx.dense())], width=32, vocab=53)
    w = fx.weights(c, 60)
    for gone in ("l0.mix.sink", "l1.mix.dq.norm", "l0.hc2.mix", "l0.norm1.alpha", "final.norm.b", "head",
                 "l0.mlp.correction", "l1.mlp.up"):
        bad = dict(w)
        del bad[gone]
        with pytest.raises(KeyError, match=gone):
            make_engine(tmp_path / "x", c, bad, "cpu", "float32")
    for extra in ("l1.mix.extra", "l0.hc3.in", "l0.mlp.e9.gate", "loose"):
        with pytest.raises(KeyError, match=extra):
            make_engine(tmp_path / "y", c, dict(w, **{extra: torch.zeros(3)}), "cpu", "float32")
    with pytest.raises(ValueError, match="l1.mix.uq"):
        make_engine(tmp_path / "z", c, dict(w, **{"l1.mix.uq": torch.zeros(7, 32)}), "cpu", "float32")


def test_a_configuration_without_streams_is_an_ordinary_residual(tmp_path):
    """No `streams` entry: one stream, no connection tensors in the checkpoint, x <- x + m y."""
    c = fx.config([(fx.latent(1), fx.moe()), (fx.latent(2), fx.dense())], width=32, vocab=53, streams=1)
    w = fx.weights(c, 61)
    ones = {k: torch.ones_like(v) for k, v in w.items() if ".hc" in k}
    toks = tokens(19, c["vocab"], 62)
    want = Expected(c, dict(w, **ones), toks)
    plain = {k: v for k, v in c.items() if k != "streams"}
    eng = make_engine(tmp_path, plain, {k: v for k, v in w.items() if ".hc" not in k}, "cpu", "float32")
    close(run_schedule(eng, {"a": toks}, [[("a", 12)], [("a", 7)]])["a"], want, "float32")
    eng.exit()


def test_engine_refuses_what_the_kernels_do_not_take(tmp_path):
    import types
    one = types.SimpleNamespace(tp_degree=1)

    def cfg(c):
        from minivllm_amd.models.danipel import DanipelConfig
        return DanipelConfig.from_dict(c)
    ok = fx.default_config()
    cfg(ok).validate_engine(one)
    with pytest.raises(ValueError, match="one rank"):
        cfg(ok).validate_engine(types.SimpleNamespace(tp_degree=2))
    for layers, kw, what in (([(fx.latent(1, kv_rank=1020), None)], {}, "1024"),
                             ([(fx.latent(1), None)], {"streams": 9}, "streams"),
                             ([(fx.latent(1), fx.moe(experts=2, identity=1, top=4))], {}, "top"),
                             ([(fx.latent(1, rot_dim=5), None)], {}, "rot.dims")):
        with pytest.raises(ValueError, match=what):
            cfg(fx.config(layers, **kw)).validate_engine(one)
    bad = fx.default_config()
    bad["layers"][0]["type"] = "latent_attention_3"
    with pytest.raises(ValueError, match="latent_attention_3"):
        cfg(bad)


def test_benchmark_configuration_parses_and_validates():
    import types
    sys.path.insert(0, ROOT)
    import bench
    for size in ("w1024", "w2048"):
        mc = bench.danipel_model(size)
        mc.validate_engine(types.SimpleNamespace(tp_degree=1))
        kinds = [L.type for L in mc.layers]
        assert len(kinds) == 8 and kinds.count("latent_attention") == 4 and mc.streams == 2
        assert [L.mlp["kind"] for L in mc.layers] == ["dense"] + ["moe"] * 7
