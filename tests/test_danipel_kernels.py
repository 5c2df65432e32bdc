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
@pytest.mark.parametrize("NE,identity,top,W,T", [(8, 2, 4, 96, 33), (5, 0, 5, 37, 3), (1, 1, 1, 8, 2), (120, 20, 9, 72, 21),
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
@pytest.mark.parametrize("C,T", [(384, 17), (37, 5), (4608, 3)])
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
@pytest.mark.parametrize("H,D,P,R,dims", [(6, 32, 32, 96, 32), (3, 10, 14, 20, 12), (8, 64, 64, 512, 64), (2, 8, 8, 8, 0)])
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
