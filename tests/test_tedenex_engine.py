"""The Tedenex family inside the engine (registry, loader, scheduler, paged caches, state slots,
kernels) against the plain oracle of ``tedenex_oracle``: every mechanism alone (one-layer models),
whole prompts and the stream after every layer run, token-by-token decoding, portions down to two
tokens, mixed batches against each request alone, blocks and state slots that are used again, keys
that stand out (at the first token, at page borders, just inside and just outside a chunk, hundreds
of positions back; in prompts and while decoding), a state that has to reach far, long decoding,
sizes that are 1 or equal, configurations drawn at random, greedy generation through
``LLMEngine.generate``, and the replay entry point.  Every test runs on the CPU (fp32); the ``gpu``
variants run the HIP kernels in float32 and bfloat16."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import tedenex_fixtures as fx
import tedenex_oracle as oracle

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
    assert type(mc).__name__ == "TedenexConfig"
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
    of the logits themselves."""
    d = got.double() - want.logits
    d = d - d.mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / want.logits.std(-1)
    if dtype == "float32":
        assert float(e.max()) < 2e-4, f"logits differ: {float(e.max()):.3g} at {int(e.argmax())}"
    else:
        assert float(e.median()) < 0.06, f"typical row differs: {float(e.median()):.3g}"
        assert float(e.max()) < 0.25, f"logits differ: {float(e.max()):.3g} at {int(e.argmax())}"


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
    "attention": ([(fx.attention(), None)], None),
    "attention-one-tap": ([(fx.attention(conv=1), None)], None),
    "attention-two-taps": ([(fx.attention(dim=16, vdim=8, conv=2), None)], None),
    "attention-many-taps": ([(fx.attention(conv=7, size=5), None)], None),
    "attention-runs-of-eight": ([(fx.attention(heads=6, kv_heads=2, dim=24, vdim=40, conv=4, size=13), None)], None),
    "attention-serving-sizes": ([(fx.attention(heads=8, kv_heads=2, dim=64, vdim=128, conv=4, size=16, scale=0.1), None)], None),
    "attention-long-heads": ([(fx.attention(heads=2, kv_heads=1, dim=320, vdim=264, conv=3, size=20, scale=0.05), None)], None),
    "wkv": ([(fx.wkv(), None)], None),
    "wkv-serving-sizes": ([(fx.wkv(heads=4, dim=64), None)], None),
    "wkv-wide": ([(fx.wkv(heads=1, dim=130), None)], None),
    "latent": ([(fx.latent(), None)], None),
    "latent-serving-sizes": ([(fx.latent(heads=16, dim=64, rot_dim=64, vdim=64, kv_rank=128, q_rank=48, scale=0.09), None)], None),
    "dense": ([(fx.wkv(), fx.dense())], None),
    "loop": ([(fx.wkv(), None), (fx.attention(), None)], (0, 2, 3)),
    "loop-one-layer": ([(fx.latent(), None), (fx.attention(), fx.dense())], (1, 2, 2)),
    "loop-once": ([(fx.wkv(), None), (fx.latent(), None)], (0, 1, 1)),
}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", list(ALONE))
def test_each_mechanism_alone(tmp_path, device, dtype, kind):
    """Whole prompt, then the same tokens as prompt portions + single tokens."""
    layers, loop = ALONE[kind]
    c = fx.config(layers, width=32, vocab=53, loop=loop)
    w = fx.weights(c, 40)
    toks = tokens(33, c["vocab"], 41)
    eng = make_engine(tmp_path, c, w, device, dtype)
    seen = []
    eng.model_runner.model.model.layer_hook = lambda i, x: seen.append(x.detach().float().cpu().clone())
    want = Expected(c, w, toks)
    close(run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"], want, dtype)
    lim, n = 1e-4 if dtype == "float32" else 0.1, len(toks)
    assert len(seen) == len(want.trace)
    for x, ref in zip(seen, want.trace):
        assert float((x[:n].double() - ref).abs().max()) < lim * float(ref.abs().max())
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
    assert len(seen) == len(oracle.run_order(c))
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
             [("a", 20), ("b", 1), ("c", 1)],              # b ends: its blocks and slot return
             [("a", 1), ("c", 1), ("d", 1)],               # d's first token alone
             [("e", 3), ("a", 1), ("c", 1)],
             [("e", 15), ("a", 9), ("c", 2)]]
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=14, seqs=3)
    got = run_schedule(eng, reqs, sched)
    for k, toks in reqs.items():
        close(got[k], Expected(c, w, toks), dtype)
    bm = eng.scheduler.block_manager
    assert bm.num_free_blocks == bm.num_blocks
    assert eng.scheduler.state_pool.num_free == 3
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_pools_used_again(tmp_path, device, dtype):
    """A KV pool of just over one request and two state slots: every later request runs on blocks
    and state rows that an earlier one has left dirty (its first tokens read zeros all the same)."""
    c = fx.default_config()
    w = fx.weights(c, 13)
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=9, seqs=2)
    for i, n in enumerate([60, 33, 64, 9, 2, 1]):
        toks = tokens(n, c["vocab"], 20 + i)
        cut = max(1, n // 3)
        got = run_schedule(eng, {"r": toks}, [[("r", cut)], [("r", n - cut)]] if n > 1 else [[("r", 1)]])["r"]
        close(got, Expected(c, w, toks), dtype)
    eng.exit()


def _swap(t):
    h = t.shape[-1] // 2
    return torch.cat([t[..., h:], t[..., :h]], -1).contiguous()


def _standout_attention(size):
    """One attention layer made so that ONE key stands out for token 39: token 38's embedding is
    token 39's with its halves swapped, head 1's key rows are its query rows with their input
    columns swapped, the filters pass the current token alone, so k(38) = q_1(39); the distance
    penalty of head 1 of 2 is small."""
    W, D = 32, 16
    c = fx.config([(fx.attention(heads=2, kv_heads=1, dim=D, vdim=D, conv=2, size=size, scale=0.8), None)],
                  width=W, vocab=40)
    w = fx.weights(c, 50)
    p = "l0.mix."
    w["l0.norm1"] = torch.zeros_like(w["l0.norm1"])
    for n in "qk":
        w[p + n + ".b"] = torch.zeros_like(w[p + n + ".b"])
        w[p + n + ".norm"] = torch.ones_like(w[p + n + ".norm"])
    for n in "qkv":                                                # (a value's filter would reach over the edge)
        w[p + n + ".conv"] = torch.tensor([[0.0, 1.0]]).expand(w[p + n].shape[0], 2).contiguous()
    w[p + "k"] = _swap(w[p + "q"][D:])
    e = w["embed"].clone()
    e[38] = _swap(e[39])
    w["embed"] = e
    return c, {k: v.to(torch.bfloat16) for k, v in w.items()}


def _standout_latent():
    """The same for one latent layer: head 1's unrotated query is a multiple of the latent of the
    swapped input, its unrotated key IS the latent; the rotated part is small."""
    W, R = 32, 16
    c = fx.config([(fx.latent(heads=2, dim=R, rot_dim=4, vdim=R, kv_rank=R, q_rank=R, scale=0.5), None)],
                  width=W, vocab=40)
    w = fx.weights(c, 50)
    p = "l0.mix."
    w["l0.norm1"] = torch.zeros_like(w["l0.norm1"])
    for n in ("dkv.norm", "dq.norm"):
        w[p + n] = torch.ones_like(w[p + n])
    uk, uq, dkv = w[p + "uk"].clone(), w[p + "uq"].clone(), w[p + "dkv"].clone()
    uk[R:2 * R] = torch.eye(R)
    uq[R + 4:2 * R + 4] = 2.0 * torch.eye(R)
    dkv[R:] = 0.3 * dkv[R:]
    w[p + "uk"], w[p + "uq"], w[p + "dkv"] = uk, uq, dkv
    w[p + "dq"] = _swap(dkv[:R])
    e = w["embed"].clone()
    e[38] = _swap(e[39])
    w["embed"] = e
    return c, {k: v.to(torch.bfloat16) for k, v in w.items()}


def _check_standout(eng, c, w, n, places, dtype, decoded, visible):
    q = n - 1
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
        moved, spread = float((want.logits[q] - without).std()), float(without.std())
        if visible(where, q):
            assert moved > 0.2 * spread, "the key does not stand out"
            if dtype == "bfloat16":
                assert float((got[q].double() - want.logits[q]).std()) < 0.3 * moved
        else:
            assert moved < 1e-9 * spread, "the key should be out of sight"


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decoded", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("n", [41, 330], ids=["short", "far"])
def test_a_latent_key_that_stands_out(tmp_path, device, dtype, decoded, n):
    """At the first token, on both sides of a page border, on both sides of the kernels' runs of
    keys (32, 64, 256), right before the query."""
    bs, q = 8, n - 1
    c, w = _standout_latent()
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=n // bs + 4, block_size=bs, seqs=2)
    places = [0, 1, bs - 1, bs, 31, 32, q - 1, q - 6] + ([63, 64, 127, 128, 255, 256] if n > 300 else [])
    _check_standout(eng, c, w, n, places, dtype, decoded, lambda j, i: True)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decoded", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("size,n", [(16, 41), (13, 40), (13, 53), (100, 330), (300, 300), (300, 301), (4096, 70)])
def test_keys_at_a_chunks_edges(tmp_path, device, dtype, decoded, size, n):
    """The first key of the query's chunk, the last one of the chunk before, the first token, page
    borders and the keys next to the query; queries in the middle of a chunk, at its end (299 of 300)
    and alone at its start (300)."""
    bs, q = 8, n - 1
    c, w = _standout_attention(size)
    lo = q // size * size
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=n // bs + 4, block_size=bs, seqs=2)
    places = {0, 1, lo - 1, lo, lo + 1, q // bs * bs - 1, q // bs * bs, q - 1} & set(range(q))
    _check_standout(eng, c, w, n, sorted(places), dtype, decoded, lambda j, i: j // size == i // size)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_chunks_count_from_the_sequences_start(tmp_path, device, dtype):
    """Portions that start and end on, just before and just behind chunk and page borders."""
    c = fx.config([(fx.attention(size=12), fx.dense()), (fx.attention(heads=2, kv_heads=1, dim=64, vdim=64, size=8,
                                                                      conv=4, scale=0.12), None)], width=32, vocab=53)
    w = fx.weights(c, 51)
    toks = tokens(61, c["vocab"], 52)
    eng = make_engine(tmp_path, c, w, device, dtype)
    want = Expected(c, w, toks)
    for cuts in ([12, 12, 13, 11, 13], [11, 2, 10, 2, 36], [8, 4, 4, 9, 36], [13, 2, 46], [59, 2]):
        got = run_schedule(eng, {"a": toks}, [[("a", n)] for n in cuts])["a"]
        close(got, want, dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decoded", [False, True], ids=["prompt", "decoded"])
def test_a_state_that_reaches_far(tmp_path, device, dtype, decoded):
    """Slow decays and strong first keys: the first token's outer product is still most of the state 150
    tokens later.  The oracle's logits for another first token differ widely."""
    c = fx.config([(fx.wkv(heads=2, dim=16), None)], width=32, vocab=53)
    w = fx.weights(c, 53)
    w["l0.mix.w0"] = torch.full_like(w["l0.mix.w0"], -7.0)
    e = w["embed"].clone()
    e[1:40] *= 0.01                                       # the tokens in between are small ...
    w["embed"] = e
    w["l0.norm1"] = torch.zeros_like(w["l0.norm1"])
    c["norm"]["eps"] = 1e-2                               # ... also behind a norm with a large eps
    n = 150
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=24)
    rows = []
    for first in (45, 50):
        toks = [first] + [1 + (t * 7) % 37 for t in range(n - 1)]
        sched = [[("a", n)]] if not decoded else [[("a", 70)]] + [[("a", 1)]] * (n - 70)
        want = Expected(c, w, toks)
        close(run_schedule(eng, {"a": toks}, sched)["a"], want, dtype)
        rows.append(want.logits[-1])
    assert float((rows[0] - rows[1]).std()) > 0.2 * float(rows[0].std())
    eng.exit()


def test_every_part_shows(tmp_path):
    """The oracle with one thing changed gives other logits than the engine: no mechanism hides
    behind the random weights."""
    c = fx.default_config()
    w = fx.weights(c, 44)
    toks = tokens(45, c["vocab"], 45)
    eng = make_engine(tmp_path, c, w, "cpu", "float32")
    got = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    close(got, Expected(c, w, toks), "float32")

    def cfg(f):
        cc = json.loads(json.dumps(c))
        f(cc)
        return cc, w

    def zero(*names):
        return c, dict(w, **{n: torch.zeros_like(w[n]) for n in names})
    last = w["l0.mix.q.conv"].clone()
    last[:, :-1] = 0
    others = [cfg(lambda k: k["layers"][0]["mixer"]["mask"].update(size=12)),
              cfg(lambda k: k["layers"][3]["mixer"]["mask"].update(size=15)),
              cfg(lambda k: k["layers"][2]["mixer"]["rot"].update(base=150.0)),
              cfg(lambda k: k["loop"].update(times=1)), cfg(lambda k: k["loop"].update(start=2)),
              zero("l0.mix.v.b"), zero("l0.mix.q.b"), zero("l1.mix.u"), zero("l4.mix.mu.w"), zero("l4.mix.mu.g"),
              zero("l1.mix.w1"), zero("l3.side.proj"), zero("l2.norm2b"), zero("l1.norm1b"),
              (c, dict(w, **{"l0.mix.q.conv": last})),
              (c, dict(w, **{"l2.side.norm": w["l2.side.norm"] + 1})),
              (c, dict(w, **{"side.embed": w["side.embed"].roll(6, 1)}))]
    for cc, ww in others:
        far = oracle.forward(cc, ww, toks)[0]
        assert float((got.double() - far).std()) > 0.005 * float(far.std())
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_decoding_over_many_blocks(tmp_path, device, dtype):
    """150 single tokens behind a prompt of three: many page and chunk borders."""
    c = fx.config([(fx.attention(heads=2, kv_heads=1, dim=8, vdim=4, size=24), fx.dense(16)), (fx.wkv(heads=2, dim=8), None),
                   (fx.latent(heads=2, dim=8, rot_dim=6, vdim=4, kv_rank=12, q_rank=8), fx.dense(16))],
                  width=24, vocab=61, loop=(0, 2, 2))
    w = fx.weights(c, 14)
    toks = tokens(150, c["vocab"], 15)
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=40, block_size=4)
    got = run_schedule(eng, {"a": toks}, [[("a", 3)]] + [[("a", 1)]] * 147)["a"]
    close(got, Expected(c, w, toks), dtype)
    eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_sizes_that_happen_to_be_one_or_equal(tmp_path, device, dtype):
    """One head, one number per head, chunks of one, a single tap, a rank of one, one number of token
    input, scales of one, every size the same, all layers in the loop."""
    for layers, extra, rank in (
            ([(fx.attention(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, size=1, scale=1.0), fx.dense(1)),
              (fx.wkv(heads=1, dim=1), None),
              (fx.latent(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1, scale=1.0), None)], dict(side=1), 1),
            ([(fx.attention(heads=4, kv_heads=4, dim=16, vdim=16, conv=4, size=16, scale=1.0), fx.dense(16)),
              (fx.wkv(heads=4, dim=16), fx.dense(16)),
              (fx.latent(heads=4, dim=16, rot_dim=16, vdim=16, kv_rank=16, q_rank=16, scale=1.0), fx.dense(16))],
             dict(side=16, loop=(0, 3, 2)), 16),
            ([(fx.attention(heads=5, kv_heads=1, dim=6, vdim=9, conv=5, size=3), None)], dict(loop=(0, 1, 4)), 2)):
        c = fx.config(layers, width=16, vocab=50, **extra)
        w = fx.weights(c, 16, rank)
        toks = tokens(21, c["vocab"], 17)
        eng = make_engine(tmp_path, c, w, device, dtype)
        got = run_schedule(eng, {"a": toks}, [[("a", 2)], [("a", 12)]] + [[("a", 1)]] * 7)["a"]
        close(got, Expected(c, w, toks), dtype)
        eng.exit()


def _random_config(seed):
    """A configuration drawn from a seed: widths, head counts and sizes (also odd ones), layer order,
    filters, chunks, ranks, the loop and constants."""
    g = torch.Generator().manual_seed(seed)

    def pick(*xs):
        return xs[int(torch.randint(0, len(xs), (1,), generator=g))]
    layers = []
    for _ in range(pick(2, 3, 4)):
        kind = pick("a", "w", "l")
        if kind == "a":
            G = pick(1, 2, 3)
            m = fx.attention(heads=G * pick(1, 2, 4), kv_heads=G, dim=pick(8, 20, 33, 56, 64), vdim=pick(8, 24, 31, 64),
                             conv=pick(1, 2, 3, 4, 6), size=pick(3, 8, 17, 64), scale=pick(0.1, 0.3))
        elif kind == "w":
            m = fx.wkv(heads=pick(1, 3, 4), dim=pick(8, 20, 33, 64))
        else:
            m = fx.latent(heads=pick(1, 3, 6, 12), dim=pick(8, 24, 64), rot_dim=pick(4, 16, 32), vdim=pick(8, 20, 64),
                          kv_rank=pick(24, 96, 128), q_rank=pick(16, 50), scale=pick(0.1, 0.2), base=pick(10.0, 10000.0, 1e6))
        layers.append((m, pick(None, fx.dense(pick(8, 40, 96)))))
    a = pick(0, 1)
    return fx.config(layers, width=pick(24, 50, 96, 160), vocab=pick(50, 131), eps=pick(1e-6, 1e-5), side=pick(3, 8, 16),
                     loop=pick(None, (a, len(layers), pick(1, 2, 3)), (0, 1, 2))), pick(2, 8, 11)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("seed", list(range(10)))
def test_configurations_drawn_at_random(tmp_path, device, dtype, seed):
    c, rank = _random_config(seed)
    w = fx.weights(c, 170 + seed, rank)
    toks = tokens(45, c["vocab"], 180 + seed)
    eng = make_engine(tmp_path, c, w, device, dtype, blocks=16, block_size=8)
    want = Expected(c, w, toks)
    close(run_schedule(eng, {"a": toks}, [[("a", 45)]])["a"], want, dtype)
    close(run_schedule(eng, {"b": toks}, [[("b", 7)], [("b", 2)], [("b", 26)]] + [[("b", 1)]] * 10)["b"], want, dtype)
    eng.exit()


def _follow(c, w, prompt, gen, dtype):
    """Greedy tokens against the oracle (recomputed from scratch per token: it keeps no state)."""
    toks = list(prompt)
    for t in gen:
        lg = oracle.forward(c, w, toks)[0][-1]
        top2 = lg.topk(2).values
        if dtype == "bfloat16" and float(top2[0] - top2[1]) < 0.15:
            break                          # a near tie: 16-bit rounding may pick either
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
def test_stateless_models_reuse_cached_prefixes(tmp_path, device, dtype):
    """Latent layers alone, looped: a block's rows of every pass are found again by prefix; with any
    state in the model every prompt is computed."""
    for layers, hits in (([(fx.latent(), fx.dense()), (fx.latent(heads=2, kv_rank=16), None)], True),
                         ([(fx.latent(), fx.dense()), (fx.attention(), None)], False)):
        c = fx.config(layers, loop=(0, 1, 2))
        w = fx.weights(c, 24)
        head = tokens(24, c["vocab"], 25)
        eng = make_engine(tmp_path, c, w, device, dtype, score=False, seqs=2, blocks=30)
        for n in (5, 7):
            prompt = head + tokens(n, c["vocab"], 26 + n)
            out = eng.generate([prompt], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
            _follow(c, w, prompt, out["token_ids"][0], dtype)
        assert (eng.scheduler.block_manager.num_prefix_hits >= 3) == hits
        eng.exit()


@pytest.mark.parametrize("device,dtype", CASES)
def test_models_of_one_mixer_kind_only(tmp_path, device, dtype):
    """Without any cache of keys (time mixing alone) and without a loop entry."""
    for layers in ([(fx.wkv(), fx.dense()), (fx.wkv(heads=1, dim=20), None)], [(fx.attention(), None), (fx.attention(), None)]):
        c = fx.config(layers)
        w = fx.weights(c, 27)
        reqs = {"a": tokens(20, c["vocab"], 28), "b": tokens(11, c["vocab"], 29)}
        eng = make_engine(tmp_path, c, w, device, dtype)
        got = run_schedule(eng, reqs, [[("a", 9)], [("a", 1), ("b", 7)], [("a", 9), ("b", 1)], [("a", 1), ("b", 3)]])
        for k, toks in reqs.items():
            close(got[k], Expected(c, w, toks), dtype)
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
    c = fx.config([(fx.attention(), fx.dense()), (fx.wkv(), None), (fx.latent(), fx.dense())], width=32, vocab=53)
    w = fx.weights(c, 60)
    for gone in ("l0.mix.q.b", "l0.mix.v.conv", "l0.mix.k.norm", "l1.mix.mu.w", "l1.mix.w0", "l2.mix.dq.norm", "l2.norm2b",
                 "l1.side.norm", "side.embed", "final.norm", "embed", "l0.mlp.up"):
        bad = dict(w)
        del bad[gone]
        with pytest.raises(KeyError, match=gone):
            make_engine(tmp_path / "x", c, bad, "cpu", "float32")
    for extra in ("l1.mix.extra", "l1.norm2", "l0.mlp.gate", "loose", "head"):
        with pytest.raises(KeyError, match=extra):
            make_engine(tmp_path / "y", c, dict(w, **{extra: torch.zeros(3)}), "cpu", "float32")
    for name in ("l2.mix.uq", "l1.mix.w2", "l0.mix.q.conv", "side.embed"):
        with pytest.raises(ValueError, match=name):
            make_engine(tmp_path / "z", c, dict(w, **{name: torch.zeros(7, 32)}), "cpu", "float32")


def test_engine_refuses_what_the_kernels_do_not_take(tmp_path):
    import types
    from minivllm_amd.models.tedenex import TedenexConfig
    one = types.SimpleNamespace(tp_degree=1)
    cfg = TedenexConfig.from_dict
    ok = fx.default_config()
    cfg(ok).validate_engine(one)
    with pytest.raises(ValueError, match="one rank"):
        cfg(ok).validate_engine(types.SimpleNamespace(tp_degree=2))
    for layer, what in ((fx.latent(kv_rank=1020), "1024"), (fx.latent(rot_dim=5), "rot.dims"), (fx.wkv(dim=257), "256"),
                        (fx.attention(heads=3, kv_heads=2), "multiple"), (fx.attention(dim=1025), "1024"),
                        (fx.attention(conv=0), "conv")):
        with pytest.raises(ValueError, match=what):
            cfg(fx.config([(layer, None)])).validate_engine(one)
    for change, what in ((lambda k: k["layers"][0].update(type="wkv2"), "wkv2"),
                         (lambda k: k["layers"][0]["mlp"].update(kind="moe"), "moe"),
                         (lambda k: k["loop"].update(stop=9), "loop")):
        bad = json.loads(json.dumps(ok))
        change(bad)
        with pytest.raises(ValueError, match=what):
            cfg(bad)


def test_benchmark_configuration_parses_and_validates():
    import types
    sys.path.insert(0, ROOT)
    import bench
    for size in ("w1024", "w2048"):
        mc = bench.tedenex_model(size)
        mc.validate_engine(types.SimpleNamespace(tp_degree=1))
        assert len(mc.run_order()) == 8 and {L.type for L in mc.layers} == {"attention", "wkv", "latent_attention"}
