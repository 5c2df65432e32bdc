"""gfx950 kernels that the Tedenex family adds or extends (``ops.hip_hybrid``) against the plain
PyTorch forms of the same ops (``ops.torch_seqmix``) on CPU copies of the same inputs: bfloat16 and
float32, sizes that are not powers of two, strided inputs, several sequences in a step (fresh ones,
ones that go on, single rows, rows of no sequence)."""
import pytest
import torch

pytestmark = pytest.mark.gpu

gpu = torch.cuda.is_available()
if gpu:
    from minivllm_amd.ops import hip_hybrid as hk
from minivllm_amd.ops import torch_seqmix as ref

DTYPES = [torch.float32, torch.bfloat16]


def tol(dt, f32=2e-5):
    return dict(rtol=2e-2, atol=2e-2) if dt == torch.bfloat16 else dict(rtol=f32, atol=f32)


def up(t):
    return None if t is None else t.cuda()


class Step:
    """Rows of a step: portions of sequences (start position, rows) in slots that others have left
    dirty, and padding rows behind them."""

    def __init__(self, portions, padding=3):
        self.n = [m for _, m in portions]
        B = len(portions)
        self.T = sum(self.n) + padding
        self.cu_q = torch.tensor([0] + self.n).cumsum(0).to(torch.int32)
        self.positions = torch.zeros(self.T, dtype=torch.int32)
        self.row_seq = torch.full((self.T,), -1, dtype=torch.int32)
        at = 0
        for b, (lo, m) in enumerate(portions):
            self.positions[at:at + m] = torch.arange(lo, lo + m)
            self.row_seq[at:at + m] = b
            at += m
        self.slots = torch.tensor(torch.randperm(B + 2)[:B].tolist(), dtype=torch.int32)
        self.num_slots, self.live = B + 2, at

    def tails(self, keep, C):
        """What filters of keep + 1 taps have left in the slots: random, zeros ahead of position 0."""
        return _tails(self.num_slots, keep, C, self.slots, self.positions[self.cu_q[:-1].long()])

    def lay(self, dev):
        return tuple(t.to(dev) for t in (self.cu_q, self.positions, self.slots))


def _tails(num, keep, C, slots, starts):
    t = torch.randn(num, keep, C)
    for s, p in zip(slots.tolist(), starts.tolist()):
        if s >= 0 and 0 < p < keep:
            t[s, :keep - p] = 0.0
    return t


MIXED = [(0, 9), (5, 1), (0, 1), (2, 2), (30, 17), (1, 3), (0, 2), (7, 6)]
LONG = [(0, 1500), (3, 1), (64, 700), (0, 2)]


def step_cases():
    return [("mixed", Step(MIXED)), ("long", Step(LONG, padding=5))]


def decode_layout(n, gaps=True):
    pos = torch.tensor([(3 * b) % 11 for b in range(n)], dtype=torch.int32)
    slots = torch.randperm(n + 3)[:n].to(torch.int32)
    if gaps:
        slots[2] = -1                                                # an unused row of a padded batch
    return pos, slots


FILTER_SIZES = [(4, 2, 16, 24, 4), (6, 3, 64, 64, 3), (2, 1, 128, 128, 4), (3, 1, 200, 136, 2), (1, 1, 512, 264, 4),
                (5, 5, 8, 8, 1), (4, 2, 10, 7, 4), (2, 1, 33, 64, 3), (4, 1, 48, 48, 6), (1, 1, 520, 16, 2)]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D,E,taps", FILTER_SIZES)
def test_filter_norm_store(dt, H, G, D, E, taps):
    torch.manual_seed(D)
    C = (H + G) * D + G * E
    w, qw, kw = torch.randn(C, taps), torch.randn(D), torch.randn(D)

    def run(mod, dev, x, tail, kc, vc, place, lay, row_seq):
        a = [t.to(dev) for t in (w, tail, qw, kw, kc, vc)]
        q = mod.conv_norm_store(x.to(dev), (H, G, D, E), a[0], a[1], a[2], a[3], 1e-4, a[4], a[5], place.to(dev),
                                *[None if t is None else t.to(dev) for t in lay],
                                **({} if mod is ref else dict(row_seq=up(row_seq))))
        return q.cpu().float(), a[1].cpu(), a[4].cpu().float(), a[5].cpu().float()
    for name, st in step_cases():
        bs = 16
        nb = st.T // bs + 2
        wide = torch.randn(st.T, C + (8 if C % 8 == 0 else 5)).to(dt)
        place = torch.randperm(nb * bs)[:st.T].to(torch.int32)
        place[3], place[st.live:] = -1, -1
        tail = st.tails(taps - 1, C)
        kc, vc = torch.zeros(nb, bs, G, D, dtype=dt), torch.zeros(nb, bs, G, E, dtype=dt)
        lay = (st.cu_q, st.positions, st.slots)
        got = run(hk, "cuda", wide, tail, kc, vc, place, lay, st.row_seq)
        want = run(ref, "cpu", wide, tail, kc, vc, place, lay, None)
        torch.testing.assert_close(got[0][:st.live], want[0][:st.live], **tol(dt, 1e-4))
        torch.testing.assert_close(got[1], want[1], rtol=0, atol=0)
        for a, b in zip(got[2:], want[2:]):
            torch.testing.assert_close(a, b, **tol(dt, 1e-4))
    n = 9
    pos, slots = decode_layout(n)
    x, tail = torch.randn(n, C).to(dt), _tails(n + 3, taps - 1, C, slots, pos)
    kc, vc = torch.zeros(2, 8, G, D, dtype=dt), torch.zeros(2, 8, G, E, dtype=dt)
    place = torch.randperm(16)[:n].to(torch.int32)
    place[2] = -1
    got = run(hk, "cuda", x, tail, kc, vc, place, (None, pos, slots), None)
    want = run(ref, "cpu", x, tail, kc, vc, place, (None, pos, slots), None)
    keep = [i for i in range(n) if i != 2]
    torch.testing.assert_close(got[0][keep], want[0][keep], **tol(dt, 1e-4))
    torch.testing.assert_close(got[1], want[1], rtol=0, atol=0)
    for a, b in zip(got[2:], want[2:]):
        torch.testing.assert_close(a, b, **tol(dt, 1e-4))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W,n", [(64, 5), (37, 5), (2056, 5), (40, 2), (1, 1)])
def test_shift_mix(dt, W, n):
    torch.manual_seed(W)
    mu = torch.rand(n, W)
    for name, st in step_cases():
        h, tail = torch.randn(st.T, W).to(dt), torch.randn(st.num_slots, 1, W)
        tg, tc = tail.cuda(), tail.clone()
        got = hk.shift_mix(h.cuda(), mu.cuda(), tg, *st.lay("cuda"), row_seq=st.row_seq.cuda())
        want = ref.shift_mix(h, mu, tc, *st.lay("cpu"))
        torch.testing.assert_close(got.cpu().float()[:, :st.live], want.float()[:, :st.live], **tol(dt))
        torch.testing.assert_close(tg.cpu(), tc, rtol=0, atol=0)
    pos, slots = decode_layout(9)
    h, tail = torch.randn(9, W).to(dt), torch.randn(12, 1, W)
    tg, tc = tail.cuda(), tail.clone()
    got = hk.shift_mix(h.cuda(), mu.cuda(), tg, None, pos.cuda(), slots.cuda())
    want = ref.shift_mix(h, mu, tc, None, pos, slots)
    keep = [i for i in range(9) if i != 2]
    torch.testing.assert_close(got.cpu().float()[:, keep], want.float()[:, keep], **tol(dt))
    torch.testing.assert_close(tg.cpu(), tc, rtol=0, atol=0)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,D", [(3, 9), (2, 32), (5, 48), (16, 64), (2, 100), (1, 200), (1, 256)])
@pytest.mark.parametrize("lpc", ["", "4", "8", "16"])
def test_wkv_scan(dt, H, D, lpc, monkeypatch):
    monkeypatch.setenv("MINIVLLM_SCAN_LPC", lpc) if lpc else monkeypatch.delenv("MINIVLLM_SCAN_LPC", raising=False)
    torch.manual_seed(D)
    bias, u = torch.randn(H * D) - 1.0, torch.randn(H, D)
    st = Step(MIXED)
    layouts = [(st.T, st.live, st.num_slots, (st.cu_q, st.positions, st.slots))]
    pos, slots = decode_layout(9)
    layouts.append((9, 9, 12, (None, pos, slots)))
    for T, live, ns, lay in layouts:
        proj = torch.randn(4, T, H * D).to(dt)
        r, k, v = (proj[i].view(T, H, D) for i in range(3))
        raw = (0.5 * torch.randn(T, H * D + 8)).to(dt)[:, :H * D]            # rows of a wider tensor
        state = torch.randn(ns, H, D, D)
        sg, sc = state.cuda(), state.clone()
        pg = proj.cuda()
        got = hk.wkv_scan(*(pg[i].view(T, H, D) for i in range(3)), raw.cuda(), bias.cuda(), u.cuda(), sg, *[up(t) for t in lay])
        want = ref.wkv_scan(r, k, v, raw, bias, u, sc, *lay)
        scale = float(want.abs().max())
        torch.testing.assert_close(got.cpu()[:live] / scale, want[:live] / scale, rtol=1e-4, atol=2e-6)
        torch.testing.assert_close(sg.cpu(), sc, rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D,E,bs,chunk", [(4, 2, 48, 48, 8, 20), (4, 1, 64, 64, 16, 96), (8, 2, 128, 128, 64, 37),
                                              (2, 1, 100, 40, 12, 128), (3, 3, 20, 260, 8, 33), (2, 1, 300, 64, 16, 50)])
def test_chunked_attention(dt, H, G, D, E, bs, chunk):
    torch.manual_seed(chunk)
    lens, qlens = [150, 37, 290, 64, 96], [150, 30, 2, 1, 40]
    B = len(lens)
    pages = [-(-n // bs) for n in lens]
    perm = torch.randperm(sum(pages) + 2).tolist()
    tables, at = torch.zeros(B, max(pages), dtype=torch.int32), 0
    for b, n in enumerate(pages):
        tables[b, :n] = torch.tensor(perm[at:at + n], dtype=torch.int32)
        at += n
    kc, vc = torch.randn(sum(pages) + 2, bs, G, D).to(dt), torch.randn(sum(pages) + 2, bs, G, E).to(dt)
    T = sum(qlens)
    q = torch.randn(T, H, D).to(dt)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])
    scale = 1.5 * D ** -0.5
    cu_q = torch.tensor([0] + qlens).cumsum(0).to(torch.int32)
    cu_k = torch.tensor([0] + lens).cumsum(0).to(torch.int32)
    pos = torch.cat([torch.arange(n - m, n) for n, m in zip(lens, qlens)]).to(torch.int32)
    row_seq = torch.repeat_interleave(torch.arange(B), torch.tensor(qlens)).to(torch.int32)
    want = torch.zeros(T, H, E)
    ref.sink_attention_prefill(q, kc, vc, cu_q, cu_k, tables, scale, None, None, want, slopes=slopes, chunk=chunk)
    got = torch.zeros(T, H, E, dtype=dt, device="cuda")
    g = (q.cuda(), kc.cuda(), vc.cuda())
    hk.sink_attention_prefill(*g, cu_q.cuda(), cu_k.cuda(), tables.cuda(), scale, None, None, got,
                              positions=pos.cuda(), max_q=max(qlens), row_seq=row_seq.cuda(), slopes=slopes.cuda(), chunk=chunk)
    torch.testing.assert_close(got.cpu().float(), want, **tol(dt, 1e-4))
    rows = torch.zeros(T, H, E, dtype=dt, device="cuda")
    hk.sink_attention_step(*g, tables.cuda(), row_seq.cuda(), pos.cuda(), scale, None, None, rows, slopes=slopes.cuda(), chunk=chunk)
    torch.testing.assert_close(rows.cpu().float(), want, **tol(dt, 1e-4))
    last = (cu_q[1:] - 1).long()
    dec = torch.zeros(B, H, E, dtype=dt, device="cuda")
    for longest in (None, max(lens)):
        hk.sink_attention_decode(q[last].contiguous().cuda(), g[1], g[2], tables.cuda(), torch.tensor(lens, dtype=torch.int32).cuda(),
                                 scale, None, None, dec, longest, slopes=slopes.cuda(), chunk=chunk)
        torch.testing.assert_close(dec.cpu().float(), want[last], **tol(dt, 1e-4))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W,T", [(40, 7), (37, 5), (1024, 33), (2048, 3), (3080, 5), (8192, 2), (8200, 2), (320, 2100)])
@pytest.mark.parametrize("plain,again", [(False, False), (True, True)])
def test_stream_update(dt, W, T, plain, again):
    torch.manual_seed(W)
    x, y = torch.randn(T, W), torch.randn(T, W + 8).to(dt)[:, :W]            # rows of a wider tensor
    wb, wn, table = torch.randn(W), torch.randn(W), torch.randn(11, W).to(dt)
    ids = torch.randint(0, 11, (T,), dtype=torch.int32)
    for kind in ("norm", "raw", "none"):
        kw = dict(plain=plain, raw=kind == "raw")
        nxt = wn if kind == "norm" else None
        xg, xc = x.cuda(), x.clone()
        got = hk.post_norm_residual(y.cuda(), wb.cuda(), xg, 1e-5, up(nxt), dt, extra=(ids.cuda(), table.cuda()) if again else None, **kw)
        want = ref.post_norm_residual(y, wb, xc, 1e-5, nxt, dt, extra=(ids, table) if again else None, **kw)
        torch.testing.assert_close(xg.cpu(), xc, rtol=2e-5, atol=2e-5)
        assert (got is None) == (want is None) == (kind == "none")
        if got is not None:
            torch.testing.assert_close(got.cpu().float(), want.float(), **tol(dt, 5e-5))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("n,T", [(392, 17), (37, 5), (4608, 3), (8, 70000)])
def test_squared_relu(dt, n, T):
    torch.manual_seed(n)
    u = (2 * torch.randn(T, n + 8)).to(dt)[:, :n]
    torch.testing.assert_close(hk.relu_squared(u.cuda(), dt).cpu().float(), ref.relu_squared(u, dt).float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("n,layers,which,T", [(24, 6, 5, 33), (7, 3, 1, 10), (256, 2, 1, 300), (1, 1, 0, 1)])
def test_token_gate(dt, n, layers, which, T):
    torch.manual_seed(n)
    z, table = (3 * torch.randn(T, n)).to(dt), torch.randn(50, n * layers).to(dt)
    ids = torch.randint(0, 50, (T,), dtype=torch.int32)
    torch.testing.assert_close(hk.token_gate(z.cuda(), ids.cuda(), table.cuda(), which * n, dt).cpu().float(),
                               ref.token_gate(z, ids, table, which * n, dt).float(), **tol(dt))


def test_steps_in_a_captured_graph():
    """Filter, shift and scan of single tokens replayed from a graph, with other tokens and slots at
    every replay, against the same steps run one by one."""
    torch.manual_seed(5)
    B, H, G, D, W, taps = 6, 4, 2, 64, 256, 4
    C = (H + 2 * G) * D
    dt = torch.bfloat16
    w, qw, kw, mu = (torch.randn(*s).cuda() for s in ((C, taps), (D,), (D,), (5, W)))
    bias, u = torch.randn(H * D).cuda(), torch.randn(H, D).cuda()
    x, h, proj = torch.zeros(B, C, dtype=dt).cuda(), torch.zeros(B, W, dtype=dt).cuda(), torch.zeros(4, B, H * D, dtype=dt).cuda()
    pos, slots, place = (torch.zeros(B, dtype=torch.int32).cuda() for _ in range(3))

    def fresh():
        return (torch.zeros(B + 2, taps - 1, C).cuda(), torch.zeros(B + 2, 1, W).cuda(), torch.zeros(B + 2, H, D, D).cuda(),
                torch.zeros(4, 8, G, D, dtype=dt).cuda(), torch.zeros(4, 8, G, D, dtype=dt).cuda())

    def step(tail, shift, state, kc, vc):
        q = hk.conv_norm_store(x, (H, G, D, D), w, tail, qw, kw, 1e-5, kc, vc, place, None, pos, slots)
        m = hk.shift_mix(h, mu, shift, None, pos, slots)
        o = hk.wkv_scan(*(proj[i].view(B, H, D) for i in range(3)), proj[3], bias, u, state, None, pos, slots)
        return q, m, o
    a, b = fresh(), fresh()
    step(*fresh())
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        outs = step(*a)
    for t in a:
        t.zero_()
    for n in range(5):
        for buf in (x, h, proj):
            buf.copy_(torch.randn(buf.shape).to(dt))
        pos.fill_(n)
        if n == 0:
            slots.copy_(torch.randperm(B).to(torch.int32))
        if n == 3:
            slots[1] = -1                                            # from here on an unused row
        place.copy_(torch.randperm(32)[:B].to(torch.int32))
        graph.replay()
        torch.cuda.synchronize()
        want = step(*b)
        live = slots >= 0
        for g_, w_ in zip(outs, want):
            if g_.shape[0] == 5:
                assert torch.equal(g_[:, live], w_[:, live])
            else:
                assert torch.equal(g_[live], w_[live])
        for s, t in zip(a, b):
            assert torch.equal(s, t)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,E,T", [(16, 64, 33), (3, 24, 7), (5, 128, 4), (2, 200, 9), (1, 512, 3), (4, 9, 5), (2, 520, 2)])
@pytest.mark.parametrize("act", ["silu", "sigmoid"])
@pytest.mark.parametrize("per_head", [True, False])
def test_gated_head_norm(dt, H, E, T, act, per_head):
    torch.manual_seed(E)
    o, w = torch.randn(T, H, E), torch.randn(H * E if per_head else E)
    gate = torch.randn(T, H * E + 8).to(dt)[:, :H * E]
    torch.testing.assert_close(hk.gated_head_norm(o.cuda(), w.cuda(), gate.cuda(), 1e-4, dt, act).cpu().float(),
                               ref.gated_head_norm(o, w, gate, 1e-4, dt, act).float(), **tol(dt))
