"""gfx950 kernels that the Danipel family adds or extends (``ops.hip_hybrid``) against the plain
PyTorch forms of the same ops (``ops.torch_seqmix``) on CPU copies of the same inputs: bfloat16
and float32, sizes that are not powers of two, strided inputs, rows that store nothing."""
import pytest
import torch

pytestmark = pytest.mark.gpu

gpu = torch.cuda.is_available()
if gpu:
    from minivllm_amd.ops import hip_hybrid as hk
from minivllm_amd.layers.rotary_embedding import HalfRotation, NeighbourRotation
from minivllm_amd.ops import torch_seqmix as ref

DTYPES = [torch.float32, torch.bfloat16]


def tol(dt, f32=2e-5):
    return dict(rtol=2e-2, atol=2e-2) if dt == torch.bfloat16 else dict(rtol=f32, atol=f32)


def up(t):
    return None if t is None else t.cuda()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("S,W,T", [(1, 40, 7), (2, 1028, 33), (3, 37, 5), (4, 2048, 9), (5, 64, 3), (8, 12, 2)])
@pytest.mark.parametrize("skip", [False, True])
def test_streams(dt, S, W, T, skip):
    torch.manual_seed(S)
    x = torch.randn(T, S, W)
    y = torch.randn(T, W + 4).to(dt)[:, :W]                        # rows of a wider tensor
    h0 = torch.randn(T, W).to(dt)
    dense = torch.rand(T, 5)
    sk = (h0, dense[:, 4]) if skip else None                       # a strided column
    write, mix, read, read2 = torch.randn(S), torch.randn(S, S), torch.randn(S), torch.randn(S)
    norm = (torch.tensor([0.8]), torch.randn(W), torch.randn(W))
    gnorm = tuple(up(t) for t in norm)
    gx, gsk = x.clone().cuda(), ((h0.cuda(), dense.cuda()[:, 4]) if skip else None)
    torch.testing.assert_close(hk.hyper_norm(gx, read.cuda(), gnorm, dt).cpu().float(),
                               ref.hyper_norm(x, read, norm, dt).float(), **tol(dt))
    row = torch.randn(T, W)
    first_g, n_g = hk.hyper_update_norm(row.cuda()[:, None, :].expand(-1, S, -1), y.cuda(), gsk, write.cuda(),
                                        mix.cuda(), read2.cuda(), gnorm, dt)
    first_c, n_c = ref.hyper_update_norm(row.clone()[:, None, :].expand(-1, S, -1), y, sk, write, mix, read2, norm, dt)
    torch.testing.assert_close(first_g.cpu(), first_c, rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(n_g.cpu().float(), n_c.float(), **tol(dt))
    out, none = hk.hyper_update_norm(gx, y.cuda(), gsk, write.cuda(), mix.cuda(), None, None, dt)
    want, _ = ref.hyper_update_norm(x, y, sk, write, mix, None, None, dt)
    assert out is gx and none is None
    torch.testing.assert_close(out.cpu(), want, rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("NE,identity,top,W,T", [(9, 3, 4, 104, 33), (5, 0, 5, 37, 3), (1, 1, 1, 8, 2), (120, 20, 9, 72, 21),
                                                 (6, 3, 2, 200, 2050)])
def test_corrected_route(dt, NE, identity, top, W, T):
    torch.manual_seed(NE)
    h = torch.randn(T, W).to(dt)
    wr, corr = torch.randn(NE + identity, W) * W ** -0.5 * 2, 0.2 * torch.randn(NE + identity)
    want = ref.corrected_route(h, wr, corr, top, identity, 1.7)
    got = hk.corrected_route(h.cuda(), wr.cuda(), corr.cuda(), top, identity, 1.7).cpu()
    near = (want - got).abs().amax(-1) > 1e-4                       # a tie that went the other way
    assert float(near.float().mean()) <= (0.002 if T > 100 else 0.0)
    torch.testing.assert_close(got.sum(-1), torch.full((T,), 1.7), rtol=1e-4, atol=1e-4)
    # exact ties go to the lower index
    tie = hk.corrected_route(h.cuda(), torch.zeros_like(wr).cuda(), torch.zeros_like(corr).cuda(), top, identity, 1.0).cpu()
    assert (tie[:, :min(top, NE)] > 0).all() and float(tie[:, min(top, NE):NE].abs().sum()) == 0.0


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("C,T", [(392, 17), (37, 5), (4608, 3)])
def test_gelu_gate(dt, C, T):
    torch.manual_seed(1)
    gu = (3 * torch.randn(T, 2 * C + 8)).to(dt)[:, :2 * C]
    torch.testing.assert_close(hk.gelu_tanh_glu(gu.cuda(), dt).cpu().float(), ref.gelu_tanh_glu(gu, dt).float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("ff,sff", [(16, 24), (3, 5)])
def test_ungated_shared_columns(dt, ff, sff):
    torch.manual_seed(2)
    T, NE = 13, 4
    dense = torch.rand(T, NE + 1)
    dense[:, 1] = 0.0
    gu = (3 * torch.randn(T, 2 * (NE * ff + sff))).to(dt)
    for gate in (True, False):
        a = ref.capped_glu_route_scale(gu, dense, ff, sff, 2.0, 1.0, dt, shared_gate=gate)
        b = hk.capped_glu_route_scale(gu.cuda(), dense.cuda(), ff, sff, 2.0, 1.0, dt, shared_gate=gate)
        torch.testing.assert_close(b.cpu().float(), a.float(), **tol(dt))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,D,P,R,dims", [(6, 24, 40, 88, 40), (3, 10, 14, 20, 12), (8, 64, 64, 512, 64), (2, 8, 8, 8, 0)])
@pytest.mark.parametrize("cls", [HalfRotation, NeighbourRotation])
def test_latent_queries_and_cache_rows(dt, H, D, P, R, dims, cls):
    torch.manual_seed(3)
    T, bs, nb = 19, 8, 5
    rot = cls(dims, 1000.0, {"factor": 3.0, "original": 100, "fast": 8.0, "slow": 1.0} if dims > 2 else None)
    q_abs = torch.randn(H, T, R).to(dt)
    proj = torch.randn(T, H * (D + P) + R + P + 16).to(dt)
    q = proj[:, :H * (D + P)].view(T, H, D + P)
    dkv = proj[:, H * (D + P) + 8:H * (D + P) + 8 + R + P]
    w, pos = torch.randn(R), torch.randint(0, 3000, (T,), dtype=torch.int32)
    slots = torch.randperm(nb * bs)[:T].to(torch.int32)
    slots[5] = -1
    res = {}
    for name, mod, to in (("cpu", ref, lambda t: t), ("gpu", hk, up)):
        cache = to(torch.zeros(nb, bs, 1, R + P, dtype=dt))
        gp = to(proj)
        qq = gp[:, :H * (D + P)].view(T, H, D + P)
        dd = gp[:, H * (D + P) + 8:H * (D + P) + 8 + R + P]
        out = mod.latent_rope_store(to(q_abs), qq, dd, to(w), 1e-5, to(pos), to(rot.inv_freq), dims, cache, None,
                                    to(slots), rot.neighbours, rot.mult)
        res[name] = (out.cpu().float(), cache.cpu().float())
    for a, b in zip(res["gpu"], res["cpu"]):
        torch.testing.assert_close(a, b, **(tol(dt) if dt == torch.bfloat16 else dict(rtol=1e-3, atol=1e-3)))


LATENT_CASES = [
    # H, R, P, block size, window: one per instance and form of the kernel, padded sizes, pages that
    # are shorter than a key tile or no divisor of it, more heads than one tile of query rows
    (16, 64, 32, 64, 0), (5, 104, 24, 32, 0), (12, 120, 40, 64, 0), (16, 128, 128, 256, 70), (3, 40, 24, 8, 0),
    (16, 256, 64, 64, 0), (5, 200, 96, 16, 33), (16, 512, 64, 64, 0), (7, 384, 128, 12, 0), (48, 128, 64, 64, 0),
    (80, 512, 64, 32, 0), (1, 8, 8, 4, 5), (128, 256, 128, 64, 100)]


@pytest.mark.parametrize("H,R,P,bs,window", LATENT_CASES)
@pytest.mark.parametrize("with_sink", [False, True])
def test_latent_attention(H, R, P, bs, window, with_sink):
    """The matrix-core kernel against the plain attention on assembled queries: portions of several
    sequences (one shorter than a tile, one that starts late, one of two tokens), then their last
    rows as single tokens with every number of context splits.  One key of the longest sequence is
    made to stand out for every query."""
    from minivllm_amd.ops import torch_seqmix
    torch.manual_seed(R + H)
    dt = torch.bfloat16
    lens, qlens = [150, 37, 290, 64], [150, 30, 2, 1]
    B, D = len(lens), R + P
    pages = [-(-n // bs) for n in lens]
    perm = torch.randperm(sum(pages) + 2).tolist()
    tables, at = torch.zeros(B, max(pages), dtype=torch.int32), 0
    for b, n in enumerate(pages):
        tables[b, :n] = torch.tensor(perm[at:at + n], dtype=torch.int32)
        at += n
    cache = torch.randn(sum(pages) + 2, bs, 1, D).to(dt)
    T = sum(qlens)
    q_abs, q_rot = torch.randn(H, T, R).to(dt), torch.randn(T, H, P).to(dt)
    far = 3                                                          # (behind every window used here)
    cache[int(tables[2, far // bs]), far % bs, 0] = torch.cat([q_abs[0, 181], q_rot[181, 0]]) * 2.0
    sink = 2.0 * torch.randn(H) if with_sink else None
    scale = 1.5 * D ** -0.5
    cu_q = torch.tensor([0, 150, 180, 182, 183], dtype=torch.int32)
    cu_k = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32)
    pos = torch.cat([torch.arange(n - m, n) for n, m in zip(lens, qlens)]).to(torch.int32)
    q = torch.cat([q_abs.transpose(0, 1), q_rot], -1)
    v = cache[..., :R]
    want = torch.zeros(T, H, R)
    torch_seqmix.sink_attention_prefill(q, cache, v, cu_q, cu_k, tables, scale, sink, None, want, window)
    assert hk.latent_attention_ok(q_abs.cuda(), cache.cuda(), P)
    gq, gr, gc, gs, gt = q_abs.cuda(), q_rot.cuda(), cache.cuda(), up(sink), tables.cuda()
    got = torch.full((T, H, R), float("nan"), dtype=dt, device="cuda")
    hk.latent_attention_prefill(gq, gr, gc, cu_q.cuda(), gt, pos.cuda(), scale, gs, got, max(qlens), window)
    torch.testing.assert_close(got.cpu().float(), want, rtol=1e-2, atol=1e-2)
    # the sequences behind the first alone, as a step with riders slices them
    part = torch.full_like(got, float("nan"))
    hk.latent_attention_prefill(gq, gr, gc, cu_q.cuda()[1:], gt[1:], pos.cuda(), scale, gs, part, max(qlens), window)
    assert torch.equal(part[150:], got[150:]) and bool(torch.isnan(part[:150]).all())
    last = (cu_q[1:] - 1).long()
    ctx = torch.tensor(lens + [0], dtype=torch.int32)                # an unused row of a padded batch
    last5 = torch.cat([last, torch.zeros(1, dtype=torch.long)])
    t5 = torch.cat([tables, torch.zeros_like(tables[:1])])
    for splits in (1, 2, 3, 8):
        dec = torch.full((5, H, R), float("nan"), dtype=dt, device="cuda")
        hk._latent(gq[:, last5].contiguous(), gr[last5].contiguous(), gc, t5.cuda(), None, None, ctx.cuda(), scale, gs,
                   dec, 5, 1, window, splits)
        torch.testing.assert_close(dec[:4].cpu().float(), want[last], rtol=1e-2, atol=1e-2)
        assert bool(torch.isnan(dec[4]).all())                       # left as it was


def test_latent_weights_keep_more_than_sixteen_bits():
    """Two keys with almost equal scores and opposite values: with weights rounded to bfloat16 the
    difference is lost altogether."""
    R, P, H = 64, 8, 2
    cache = torch.zeros(1, 64, 1, R + P, dtype=torch.bfloat16)
    cache[0, 1, 0, R] = -0.0015                                      # scores, carried by the key part alone
    cache[0, 0, 0, 0], cache[0, 1, 0, 0] = 100.0, -100.0
    q_abs = torch.zeros(H, 1, R, dtype=torch.bfloat16)
    q_rot = torch.zeros(1, H, P, dtype=torch.bfloat16)
    q_rot[..., 0] = 1.0
    p = torch.exp(cache[0, :2, 0, R].double())
    want = float(100.0 * (p[0] - p[1]) / p.sum())
    out = torch.zeros(1, H, R, dtype=torch.bfloat16, device="cuda")
    hk._latent(q_abs.cuda(), q_rot.cuda(), cache.cuda(), torch.zeros(1, 1, dtype=torch.int32, device="cuda"), None, None,
               torch.tensor([2], dtype=torch.int32, device="cuda"), 1.0, None, out, 1, 1, 0, 1)
    assert want > 0.07 and float(p[1].to(torch.bfloat16)) == 1.0
    assert abs(float(out[0, 0, 0]) - want) < 0.02 * want
