"""The ops the Danipel family adds or extends (``ops.torch_seqmix``: the engine's CPU path and the
kernels' counterpart) and the layers around them against the oracle's function for the same
mechanism, each alone, on inputs made to show what random numbers hide: a sink that dominates or
vanishes, a mix matrix that is not symmetric, a correction that overturns the scores, clamps on
both sides, YaRN ramps that begin and end inside the pairs."""
import math

import pytest
import torch

import danipel_fixtures as fx
import danipel_oracle as oracle

from minivllm_amd.layers.activation import GeluTanhAndMul
from minivllm_amd.layers.attention import LatentAttention
from minivllm_amd.layers.hyper_connection import HyperConnection
from minivllm_amd.layers.layernorm import DynamicTanh
from minivllm_amd.layers.moe import CorrectedRoutedExperts
from minivllm_amd.layers.rotary_embedding import HalfRotation, NeighbourRotation
from minivllm_amd.ops import torch_seqmix as ops
from minivllm_amd.utils.context import set_context

SCALINGS = [None, {"factor": 2.0, "original": 1000, "fast": 32.0, "slow": 1.0},
            {"factor": 8.0, "original": 64, "fast": 4.0, "slow": 0.5},
            {"factor": 1.0, "original": 64, "fast": 4.0, "slow": 1.0},
            {"factor": 3.0, "original": 20, "fast": 3.0, "slow": 3.0}]      # (no ramp: a step)


@pytest.mark.parametrize("pairs,cls", [("neighbours", NeighbourRotation), ("halves", HalfRotation)])
@pytest.mark.parametrize("scaling", SCALINGS)
@pytest.mark.parametrize("dims,n,base", [(8, 8, 100.0), (12, 14, 10000.0), (2, 2, 1e6)])
def test_rotation_layouts_and_scaling(pairs, cls, scaling, dims, n, base):
    torch.manual_seed(0)
    rot = cls(dims, base, scaling)
    x = torch.randn(300, 3, n)
    got = ops._rotate(x, torch.arange(300), rot.inv_freq, dims, rot.neighbours, rot.mult)
    want = oracle.turn(x.double(), {"dims": dims, "base": base, "scaling": scaling}, pairs)
    torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)


def test_yarn_keeps_fast_pairs_and_slows_the_last():
    sc = {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}
    plain, scaled = HalfRotation(64, 10000.0), HalfRotation(64, 10000.0, sc)
    ratio = scaled.inv_freq / plain.inv_freq
    assert float(ratio[0]) == 1.0 and abs(float(ratio[-1]) - 0.25) < 1e-6
    assert ((ratio > 0.3) & (ratio < 0.95)).any()                 # the ramp between
    assert abs(scaled.mult - (0.1 * math.log(4.0) + 1.0)) < 1e-12 and plain.mult == 1.0


def _attend(m, kind, h, w, eps, bs=4, singles=3):
    """Through the layer: pages of ``bs`` tokens in scattered order, the prompt as one portion, then
    its last rows again one by one (decode form)."""
    T = h.shape[0]
    H, D, P, E, R = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    second = kind == "latent_attention_2"
    rot = (HalfRotation if second else NeighbourRotation)(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    a = LatentAttention(H, D, P, E, R, m["scale"], 0, rot, eps, sink=not second)
    a.latent_norm.copy_(w["dkv.norm"])
    a.load_expansions(w["uk"], w["uv"], h)
    if not second:
        a.core.sink.copy_(w["sink"])
    n = -(-T // bs) + 1
    a.core.k_cache = torch.full((n, bs, 1, R + P), 9.0)
    a.core.v_cache = a.core.k_cache[..., :R]
    table = torch.arange(n - 1, -1, -1, dtype=torch.int32)[None, :]
    slots = torch.tensor([int(table[0, t // bs]) * bs + t % bs for t in range(T)], dtype=torch.int32)
    pos = torch.arange(T, dtype=torch.int32)
    if second:
        q = ops.rms_norm_rows(h @ w["dq"].T, w["dq.norm"], eps, torch.float32) @ w["uq"].T
    else:
        q = h @ w["q"].T
    q, dkv = q.view(T, H, D + P), h @ w["dkv"].T
    set_context(is_prefill=True, cu_seqlens_q=torch.tensor([0, T], dtype=torch.int32),
                cu_seqlens_k=torch.tensor([0, T], dtype=torch.int32), positions=pos, slot_mapping=slots,
                block_tables=table, row_seq=torch.zeros(T, dtype=torch.int32), num_seqs=1)
    whole = a(q, dkv).reshape(T, H * E) @ w["o"].T
    rows = []
    for t in range(T - singles, T):
        set_context(is_prefill=False, positions=pos[t:t + 1], slot_mapping=slots[t:t + 1], block_tables=table,
                    context_lens=torch.tensor([t + 1], dtype=torch.int32), num_seqs=1)
        rows.append(a(q[t:t + 1], dkv[t:t + 1]).reshape(1, H * E) @ w["o"].T)
    return whole, torch.cat(rows)


@pytest.mark.parametrize("kind,sink", [(1, -30.0), (1, 0.0), (1, 8.0), (2, None)])
@pytest.mark.parametrize("scaling", [None, fx.YARN])
@pytest.mark.parametrize("sizes", [dict(), dict(heads=1, dim=2, rot_dim=2, vdim=1, kv_rank=3, q_rank=1),
                                   dict(heads=5, dim=24, rot_dim=16, vdim=7, kv_rank=40, q_rank=64)])
def test_latent_attention_through_pages(kind, sink, scaling, sizes):
    layer = fx.latent(kind, scaling=scaling, **sizes)
    m, W, T = layer["mixer"], 18, 27
    torch.manual_seed(3)
    w = {n: torch.randn(s) * (s[-1] ** -0.5 if len(s) > 1 else 1.0) * (2.0 if n in ("q", "uq") else 1.0)
         for n, s in fx.mixer_shapes(layer["type"], m, W)}
    if kind == 1:
        w["sink"] = w["sink"] * 0.1 + sink
    h = torch.randn(T, W)
    want = oracle.latent_attention(h.double(), {k: v.double() for k, v in w.items()}, m, layer["type"], 1e-5)
    whole, last = _attend(m, layer["type"], h, w, 1e-5)
    torch.testing.assert_close(whole.double(), want, rtol=1e-4, atol=1e-4)
    torch.testing.assert_close(last.double(), want[-3:], rtol=1e-4, atol=1e-4)


def test_a_large_sink_takes_the_weight():
    torch.manual_seed(4)
    s = torch.randn(2, 3, 5, dtype=torch.float64)
    p = oracle.softmax_with_sink(s, torch.tensor([[[-60.0]], [[9.0]]], dtype=torch.float64))
    assert float((p[0].sum(-1) - 1).abs().max()) < 1e-12 and float(p[1].sum(-1).max()) < 0.1


@pytest.mark.parametrize("S", [1, 2, 3, 5, 8])
def test_streams_update_read_and_norm(S):
    torch.manual_seed(5)
    T, W, m = 11, 14, 0.7
    norm, conn = DynamicTanh(W), HyperConnection(S, m)
    alpha, w, b = torch.tensor(1.3), torch.randn(W), torch.randn(W)
    norm.alpha.copy_(alpha.reshape(1)), norm.weight.copy_(w), norm.bias.copy_(b)
    read, write, mix = torch.randn(S), torch.randn(S), torch.randn(S, S)
    conn.load(read, write, mix)
    read2 = torch.randn(S)
    x, y, h0, g = torch.randn(T, S, W), torch.randn(T, W), torch.randn(T, W), torch.rand(T)
    old = [x[:, s].double().clone() for s in range(S)]
    got_u = ops.hyper_norm(x, conn.read, norm.parts, torch.float32)
    want_u = oracle.tanh_norm(sum(read[s].double() * old[s] for s in range(S)), alpha.double(), w.double(), b.double())
    torch.testing.assert_close(got_u.double(), want_u, rtol=1e-5, atol=1e-5)
    joined = y.double() + g.double()[:, None] * h0.double()
    want = oracle.hyper_step(old, lambda u: joined, read.double(), write.double(), mix.double(), m)
    out, nxt = ops.hyper_update_norm(x, y, (h0, g), conn.write, conn.mix, read2, norm.parts, torch.float32)
    assert out is x                                               # in place
    torch.testing.assert_close(out.double(), torch.stack(want, 1), rtol=1e-5, atol=1e-5)
    want_n = oracle.tanh_norm(sum(read2[s].double() * want[s] for s in range(S)), alpha.double(), w.double(), b.double())
    torch.testing.assert_close(nxt.double(), want_n, rtol=1e-5, atol=1e-4)
    # the start: S streams that are one row, nothing joining the output, no next input
    row = torch.randn(T, W)
    keep = row.clone()
    first, none = ops.hyper_update_norm(row[:, None, :].expand(-1, S, -1), y, None, conn.write, conn.mix, None, None,
                                        torch.float32)
    want = oracle.hyper_step([keep.double()] * S, lambda u: y.double(), read.double(), write.double(), mix.double(), m)
    assert none is None and first.shape == (T, S, W)
    torch.testing.assert_close(first.double(), torch.stack(want, 1), rtol=1e-5, atol=1e-5)


def test_the_mix_is_indexed_from_to():
    x = torch.tensor([[[1.0], [10.0]]])
    mix = torch.tensor([[1.0, 3.0], [0.0, 1.0]])                  # stream 0 flows into stream 1, not back
    out, _ = ops.hyper_update_norm(x, torch.zeros(1, 1), None, torch.zeros(2), mix, None, None, torch.float32)
    assert out.flatten().tolist() == [1.0, 13.0]


def test_one_stream_with_unit_numbers_is_the_residual_sum():
    conn = HyperConnection(1, 0.5)
    x, y = torch.randn(4, 1, 6), torch.randn(4, 6)
    want = x[:, 0] + 0.5 * y
    out, _ = ops.hyper_update_norm(x, y, None, conn.write, conn.mix, None, None, torch.float32)
    torch.testing.assert_close(out[:, 0], want)
    with pytest.raises(ValueError, match="streams"):
        HyperConnection(9)


def _experts(W, f, w):
    sh = f.get("shared") or {}
    r = f["router"]
    layer = CorrectedRoutedExperts(W, f["expert"]["ff"], r["experts"], r["identity"], r["top"], f["expert"]["limit"],
                                   r["scale"], sh.get("ff", 0), sh.get("limit", 0.0))
    names = [f"e{e}" for e in range(r["experts"])] + (["shared"] if sh else [])
    layer.gate_up.copy_(torch.cat([w[n + ".gate"] for n in names] + [w[n + ".up"] for n in names], 0))
    layer.down.copy_(torch.cat([w[n + ".down"] for n in names], 1))
    layer.router.copy_(w["router"])
    layer.correction.copy_(w["correction"])
    return layer


@pytest.mark.parametrize("f", [fx.moe(), fx.moe(experts=4, identity=0, top=4), fx.moe(experts=3, identity=5, top=6),
                               fx.moe(experts=6, identity=1, top=1, scale=1.0, shared_ff=0),
                               fx.moe(experts=1, identity=1, top=2, ff=4, limit=0.3, shared_ff=4, shared_limit=3.0)])
def test_routed_experts_against_the_oracle(f):
    torch.manual_seed(6)
    T, W = 23, 12
    w = {n: torch.randn(s) for n, s in fx.ff_shapes(f, W)}
    w["correction"] = 0.3 * w["correction"]
    h = torch.randn(T, W)
    want = oracle.routed_ff(h.double(), {k: v.double() for k, v in w.items()}, f)
    y, skip = _experts(W, f, w)(h)
    got = y if skip is None else y + skip[1][:, None] * skip[0]
    assert (skip is None) == (f["router"]["identity"] == 0)
    torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)


def test_the_correction_chooses_but_does_not_weigh():
    """Expert 0 has the largest score everywhere; the correction bars it and lifts expert 3: the
    chosen weights are the uncorrected scores of 3 and of the best other one, renormalised."""
    h = torch.ones(1, 2)
    router = torch.tensor([[2.0, 0.0], [1.0, 0.0], [0.5, 0.0], [-1.0, 0.0], [0.0, 0.0]])
    corr = torch.tensor([-5.0, 0.0, 0.0, 5.0, 0.0])
    d = ops.corrected_route(h, router, corr, 2, 1, 2.5)
    s = torch.softmax(router[:, 0], -1)
    assert d.shape == (1, 5)
    torch.testing.assert_close(d[0], torch.stack([s[0] * 0, s[1], s[2] * 0, s[3], s[4] * 0]) / (s[1] + s[3]) * 2.5)
    # the identity expert lifted instead: its weight lands in the last column
    d = ops.corrected_route(h, router, torch.tensor([0.0, 0.0, 0.0, 0.0, 5.0]), 2, 1, 1.0)
    torch.testing.assert_close(d[0, 4], s[4] / (s[0] + s[4]))
    # exact ties: the lower index
    d = ops.corrected_route(h, torch.zeros(4, 2), torch.zeros(4), 2, 2, 1.0)
    assert d[0].tolist() == [0.5, 0.5, 0.0]


def test_gelu_gate_and_ungated_shared_columns():
    torch.manual_seed(7)
    gu = 3 * torch.randn(9, 20)
    got = GeluTanhAndMul()(gu)
    torch.testing.assert_close(got.double(), oracle.gelu_tanh(gu[:, :10].double()) * gu[:, 10:].double(),
                               rtol=1e-5, atol=1e-5)
    # a dense matrix with one more column than experts: a gate of the shared columns or not
    dense = torch.tensor([[0.0, 0.25]])
    gu = torch.ones(1, 8)
    gated = ops.capped_glu_route_scale(gu, dense, 2, 2, 5.0, 5.0, torch.float32)
    plain = ops.capped_glu_route_scale(gu, dense, 2, 2, 5.0, 5.0, torch.float32, shared_gate=False)
    assert gated[0, :2].tolist() == [0.0, 0.0] and plain[0, :2].tolist() == [0.0, 0.0]
    torch.testing.assert_close(gated[0, 2:], 0.25 * plain[0, 2:])


def test_the_clamps_bite_on_both_sides():
    g = torch.tensor([[-9.0, 0.5, 9.0, 9.0]])
    u = torch.tensor([[9.0, -9.0, 0.25, -0.25]])
    eye = torch.eye(4)
    want = oracle.capped_expert(torch.ones(1, 1).double(), g.T.double(), u.T.double(), eye.double(), 2.0)
    got = ops.capped_glu_route_scale(torch.cat([g, u], 1), torch.ones(1, 2), 4, 0, 2.0, 0.0, torch.float32,
                                     shared_gate=False)
    torch.testing.assert_close(got.double(), want, rtol=1e-5, atol=1e-6)
