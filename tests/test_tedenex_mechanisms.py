"""Mechanisms of the Tedenex family on the CPU, each against its plain form in ``tedenex_oracle``: the
ops and layers alone, with inputs made so that a fault shows."""
import pytest
import torch

import tedenex_oracle as oracle

from minivllm_amd import ops
from minivllm_amd.layers.attention import FilteredHeads, SinkAttention
from minivllm_amd.layers.embedding_head import LayerTokenInput, ScaledTiedHead
from minivllm_amd.layers.linear_attention import TokenShiftWKV
from minivllm_amd.models.tedenex import TedenexConfig
from minivllm_amd.utils.context import reset_context, set_context

F64 = torch.float64


def near(a, b, tol=2e-5):
    torch.testing.assert_close(a.double(), b.double(), rtol=tol, atol=tol)


def steps_of(n, cuts):
    at = 0
    for m in cuts:
        yield at, m
        at += m
    assert at == n


def prefill_context(lo, m, slot, **kw):
    set_context(True, cu_seqlens_q=torch.tensor([0, m], dtype=torch.int32),
                cu_seqlens_k=torch.tensor([0, lo + m], dtype=torch.int32), num_seqs=1, max_seqlen_q=m,
                positions=torch.arange(lo, lo + m, dtype=torch.int32), state_slots=torch.tensor([slot], dtype=torch.int32),
                row_seq=torch.zeros(m, dtype=torch.int32), **kw)


@pytest.mark.parametrize("taps", [1, 2, 4, 9])
@pytest.mark.parametrize("cuts", [[23], [1] * 23, [2, 2, 5, 1, 13], [3, 20]])
def test_filter_norm_and_store(taps, cuts):
    H, G, D, E, n, bs, slot = 4, 2, 5, 7, 23, 4, 1
    C = (H + G) * D + G * E
    torch.manual_seed(taps)
    m = FilteredHeads(H, G, D, E, taps, 1e-4)
    core = SinkAttention(H, G, D, E, 1.0, sink=False)
    m.conv_weight.copy_(torch.randn(C, taps))
    m.q_norm.copy_(torch.randn(D))
    m.k_norm.copy_(torch.randn(D))
    m.slots[0].conv_state = torch.full((3, taps - 1, C), 1e6)            # a slot somebody else has left
    core.k_cache, core.v_cache = torch.zeros(8, bs, G, D), torch.zeros(8, bs, G, E)
    x = torch.randn(n, C + 3)
    place = torch.randperm(8 * bs)[:n].to(torch.int32)
    place[4] = -1
    q = []
    for lo, k in steps_of(n, cuts):
        prefill_context(lo, k, slot, slot_mapping=place[lo:lo + k])
        q.append(m(x[lo:lo + k], core))
    reset_context()
    y = oracle.time_filter(x[:, :C].to(F64), m.conv_weight.to(F64))
    near(torch.cat(q), oracle.unit_rms(y[:, :H * D].view(n, H, D), 1e-4) * m.q_norm.double())
    k = oracle.unit_rms(y[:, H * D:(H + G) * D].view(n, G, D), 1e-4) * m.k_norm.double()
    for t in range(n):
        p = int(place[t])
        if p >= 0:
            near(core.k_cache[p // bs, p % bs], k[t])
            near(core.v_cache[p // bs, p % bs], y[t, (H + G) * D:].view(G, E))
    assert float(m.slots[0].conv_state[[0, 2]].min() if taps > 1 else 1e6) == 1e6    # other slots untouched


@pytest.mark.parametrize("cuts", [[17], [1] * 17, [2, 2, 13], [5, 1, 11]])
@pytest.mark.parametrize("D", [4, 33])
def test_time_mixing(cuts, D):
    W, H, n, eps, rank = 12, 3, 17, 1e-3, 5
    g = torch.Generator().manual_seed(D)

    def rnd(*s):
        return torch.randn(*s, generator=g)
    w = {"mu." + k: 0.5 + 0.5 * rnd(W) for k in "rkvgw"}
    w.update({k: rnd(H * D, W) * W ** -0.5 for k in "rkvg"})
    w.update(w1=rnd(rank, W), w2=rnd(H * D, rank), w0=rnd(H * D) - 1, u=rnd(H, D), norm=1 + 0.2 * rnd(H * D),
             o=torch.eye(H * D))
    h = rnd(n, W)
    u = TokenShiftWKV(W, H, D, eps, passes=2)
    u.mu.copy_(torch.stack([w["mu." + k] for k in "rkvgw"]))
    u.proj.copy_(torch.stack([w[k].t() for k in "rkvg"]))
    u.decay_down.data, u.decay_up.data = w["w1"], w["w2"]
    u.decay_bias.copy_(w["w0"])
    u.bonus.copy_(w["u"])
    u.norm_weight.copy_(w["norm"])
    for st in u.slots:
        st.state, st.shift = torch.full((2, H, D, D), 1e6), torch.full((2, 1, W), 1e6)
    got = []
    for lo, k in steps_of(n, cuts):
        prefill_context(lo, k, 0)
        got.append(u(h[lo:lo + k], 1))
    reset_context()
    want = oracle.wkv(h.to(F64), {k: v.to(F64) for k, v in w.items()}, {"heads": H, "dim": D}, eps)
    near(torch.cat(got), want, 2e-4)
    assert float(u.slots[0].state.min()) == 1e6 and float(u.slots[1].state[1].min()) == 1e6


def test_bonus_counts_for_the_current_token_alone():
    """Without decay and with orthogonal keys: token t's own product enters its output times u and
    every later output once."""
    D = 4
    r, k = torch.ones(3, 1, D), torch.eye(D)[:3].view(3, 1, D)
    v = torch.tensor([1.0, 10.0, 100.0]).view(3, 1, 1).expand(3, 1, D).contiguous()
    raw = torch.full((3, D), -60.0)                                      # w = exp(-exp(-60)) = 1
    state = torch.zeros(1, 1, D, D)
    lay = (torch.tensor([0, 3], dtype=torch.int32), torch.arange(3, dtype=torch.int32), torch.zeros(1, dtype=torch.int32))
    o = ops.wkv_scan(r, k, v, raw, torch.zeros(D), torch.full((1, D), 5.0), state, *lay)
    near(o[:, 0, 0], torch.tensor([5.0, 1 + 50.0, 11 + 500.0]))
    gone = ops.wkv_scan(r, k, v, raw + 70, torch.zeros(D), torch.full((1, D), 5.0), state, *lay)   # w = 0
    near(gone[:, 0, 0], torch.tensor([5.0, 50.0 + 1.0, 500.0 + 10.0]))


@pytest.mark.parametrize("size", [1, 5, 8, 100])
def test_chunked_attention_with_a_distance_penalty(size):
    H, G, D, E, n, bs = 4, 2, 6, 5, 29, 8
    torch.manual_seed(size)
    q, k, v = torch.randn(n, H, D), torch.randn(n, G, D), torch.randn(n, G, E)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])
    kc, vc = torch.zeros(4, bs, G, D), torch.zeros(4, bs, G, E)
    kc.view(-1, G, D)[:n], vc.view(-1, G, E)[:n] = k, v
    table = torch.arange(4, dtype=torch.int32)[None]
    want = torch.zeros(n, H, E, dtype=F64)
    for i in range(n):
        for h in range(H):
            js = [j for j in range(i + 1) if j // size == i // size]
            s = torch.stack([0.7 * (q[i, h].double() @ k[j, h // 2].double()) - float(slopes[h]) * (i - j) for j in js])
            want[i, h] = torch.softmax(s, 0) @ v[js, h // 2].double()
    out = torch.zeros(n, H, E)
    ops.sink_attention_prefill(q, kc, vc, torch.tensor([0, n]), torch.tensor([0, n]), table, 0.7, None, None, out,
                               slopes=slopes, chunk=size)
    near(out, want)
    for i in range(n):
        o1 = torch.zeros(1, H, E)
        ops.sink_attention_decode(q[i:i + 1], kc, vc, table, torch.tensor([i + 1]), 0.7, None, None, o1,
                                  slopes=slopes, chunk=size)
        near(o1[0], want[i])
    with pytest.raises(ValueError, match="chunks"):
        SinkAttention(H, G, D, E, 1.0, chunk=4, window=8, keep_first=1)


@pytest.mark.parametrize("plain", [False, True])
@pytest.mark.parametrize("again", [False, True])
def test_stream_update(plain, again):
    torch.manual_seed(1)
    T, W, eps = 5, 13, 1e-2
    x, y, w, wn, table = torch.randn(T, W), 0.1 * torch.randn(T, W), torch.randn(W), torch.randn(W), torch.randn(7, W)
    ids = torch.tensor([6, 0, 3, 3, 1], dtype=torch.int32)
    want = x.double() + oracle.unit_rms(y.double(), eps) * (w.double() if plain else 1 + w.double())
    if again:
        want = want + table[ids.long()].double()
    for kind in ("norm", "raw", "none"):
        xx = x.clone()
        h = ops.post_norm_residual(y, w, xx, eps, wn if kind == "norm" else None, torch.float32, plain=plain,
                                   raw=kind == "raw", extra=(ids, table) if again else None)
        near(xx, want)
        if kind == "none":
            assert h is None
        else:
            near(h, want if kind == "raw" else oracle.unit_rms(want, eps) * (1 + wn.double()))


def test_token_input_takes_its_own_run():
    torch.manual_seed(2)
    T, W, n, layers = 4, 10, 3, 4
    table, ids = torch.randn(9, n * layers), torch.tensor([8, 1, 1, 0], dtype=torch.int32)
    x = torch.randn(T, W)
    for i in range(layers):
        m = LayerTokenInput(W, n, i * n)
        m.gate.copy_(torch.randn(n, W))
        m.proj.copy_(torch.randn(W, n))
        want = oracle.token_input(x.double(), table[ids.long()][:, i * n:(i + 1) * n].double(),
                                  {"gate": m.gate.double(), "proj": m.proj.double(), "norm": torch.ones(W, dtype=F64)}, 1e-3)
        near(oracle.unit_rms(m(x, ids, table).double(), 1e-3), want, 1e-4)


def test_squared_relu_and_head():
    z = torch.tensor([[-3.0, -0.5, 0.0, 0.5, 3.0, 7.0]])
    near(ops.relu_squared(z[:, 1:5], torch.float32), torch.tensor([[0.0, 0.0, 0.25, 9.0]]))
    emb = torch.nn.Embedding(5, 4)
    head = ScaledTiedHead(emb, 1e-3, offset=1.0)
    w, x = torch.randn(4), torch.randn(3, 4)
    head.load_norm(w)
    reset_context()
    near(head(x).detach(), oracle.unit_rms(x.double(), 1e-3) * (1 + w.double()) @ emb.weight.detach().double().T)


def test_run_order_of_loops():
    def order(n, loop):
        c = TedenexConfig(10, 8, [None] * n)
        if loop:
            c.loop_start, c.loop_stop, c.loop_times = loop
        return c.run_order()
    assert order(3, None) == [(0, 0, False), (1, 0, False), (2, 0, False)]
    assert order(3, (1, 2, 3)) == [(0, 0, False), (1, 0, False), (1, 1, True), (1, 2, True), (2, 0, False)]
    assert order(2, (0, 2, 2)) == [(0, 0, False), (1, 0, False), (0, 1, True), (1, 1, False)]
    assert order(2, (0, 2, 1)) == [(0, 0, False), (1, 0, False)]
