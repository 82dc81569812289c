"""The Monolix kernels at the layer sizes of real models (bf16 and fp32), each against a plain fp32 torch expression of the
same operation evaluated on the GPU: several requests of unequal length in one launch.  Every case prints its name before it
launches."""
import pytest
import torch

from tests.test_gpu_toredra_kernels import DEV, announce, close, rms, seq_extend

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 2e-5), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("T", [8, 4096])
def test_mixture_join_at_model_size(dtype, bar, T):
    from scratchpad_amd import _native
    W, top, E, outputs = 4096, 6, 64, 96
    announce("post_norm with a mixture", dtype, "rows", T)
    g = torch.Generator(device=DEV).manual_seed(1)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    x, a, z = rn(T, W), rn(T, W).to(dtype), rn(T * top, W).to(dtype)
    weight, scale, gate = rn(W) * 0.2 + 1, rn(W) * 0.2 + 1, torch.rand(T, generator=g, device=DEV)
    ids = torch.rand(T, outputs, generator=g, device=DEV).topk(top)[1].to(torch.int32)
    wts = torch.rand(T, top, generator=g, device=DEV)
    place = torch.randperm(T * top, generator=g, device=DEV).to(torch.int32)
    y = gate[:, None] * a.float()
    for k in range(top):
        row = z[place.view(T, top)[:, k].long()].float()
        y += wts[:, k:k + 1] * torch.where((ids[:, k:k + 1] >= E), x, row)
    want = rms(3.0 * x + scale * y, 1e-5) * weight
    xs = x.clone()
    lo = _native.post_norm(xs, a, weight, 1e-5, 3.0, dtype, scale=scale, z=z, ids=ids, place=place, weights=wts, gate=gate, experts=E)
    close(xs, want, 2e-5)
    close(lo, want, bar)


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 1e-4), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,G,D,dims", [(16, 4, 128, 64), (32, 8, 64, 64), (8, 8, 256, 32)])
def test_attention_on_keys_at_model_size(dtype, bar, H, G, D, dims):
    from scratchpad_amd import _native
    from scratchpad_amd.layers import HalfAngleRotary
    lens, slots = [700, 1, 323], [3, 1, 4]
    T = sum(lens)
    announce("keys as values", dtype, "heads", H, "kv heads", G, "dim", D, "tokens", lens)
    g = torch.Generator(device=DEV).manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    qk, qb, kb, qn, kn = rn(T, (H + G) * D).to(dtype), rn(H * D) * 0.3, rn(G * D) * 0.3, 1 + 0.3 * rn(D), 1 + 0.3 * rn(D)
    rot = HalfAngleRotary(dims, 10000.0).to(DEV)
    pos = torch.cat([torch.arange(m, device=DEV) for m in lens])
    loc = torch.randperm(T, generator=g, device=DEV) + 1
    table = torch.zeros(6, 800, dtype=torch.int32, device=DEV)
    kpool, vpool = (torch.full((T + 1, G * D), float("nan"), dtype=dtype, device=DEV) for _ in range(2))
    want, at = torch.empty(T, H, D, device=DEV), 0
    half = dims // 2

    def make(z, nw):                                           # [m, heads, D] -> normed, rotated
        z = rms(z, 1e-5) * nw
        ang = torch.arange(z.shape[0], device=DEV).float()[:, None] * rot.freq
        c, s = ang.cos()[:, None], ang.sin()[:, None]
        u, v = z[..., :half], z[..., half:dims]
        return torch.cat([u * c - v * s, v * c + u * s, z[..., dims:]], -1)
    for m, slot in zip(lens, slots):
        table[slot, :m] = loc[at:at + m].to(torch.int32)
        q = make(qk[at:at + m, :H * D].float().add(qb).view(m, H, D), qn)
        k0 = qk[at:at + m, H * D:].float().add(kb).view(m, G, D)
        k = make(k0, kn).repeat_interleave(H // G, 1)
        s = torch.matmul(q.transpose(0, 1), k.permute(1, 2, 0).contiguous()) * 0.09
        s = s.masked_fill(~torch.ones(m, m, dtype=torch.bool, device=DEV).tril(), float("-inf"))
        want[at:at + m] = torch.matmul(s.softmax(-1), k0.repeat_interleave(H // G, 1).transpose(0, 1).contiguous()).transpose(0, 1)
        at += m
    q = qk[:, :H * D]
    _native.qkv_rotary_store(q, qk[:, H * D:], None, kpool, vpool, pos, loc, rot.freq, 1.0, H, G, D, D, 1e-5, norm_values=False,
                             q_bias=qb, k_bias=kb, qk_norm=2, q_norm_weight=qn, k_norm_weight=kn)
    got = _native.window_attention(q, kpool, vpool, None, None, table, seq_extend(lens, [0, 0, 0], slots), H, G, D, D, 0, 0, 0.09)
    close(got, want.reshape(T, H * D), bar)


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 1e-4), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("T", [8, 1024])
def test_identity_mixture_at_model_size(dtype, bar, T):
    from scratchpad_amd.layers import PostNorm
    from scratchpad_amd.moe import IdentityMoE
    W, E, ident, top, ff = 2048, 32, 8, 4, 1024
    announce("IdentityMoE + PostNorm", dtype, "rows", T)
    g = torch.Generator(device=DEV).manual_seed(2)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    with torch.device(DEV):
        mlp, norm = IdentityMoE(W, E, ident, top, ff, 4, 2, shared_ff=W, dtype=dtype), PostNorm(W, 1e-5, 3.0, layer_scale=True)
    for p in (mlp.experts.up, mlp.experts.down, mlp.shared.up, mlp.shared.down, mlp.router.weight):
        p.data.copy_(rn(*p.shape) * p.shape[-1] ** -0.5)
    mlp.router.correction.data.copy_(rn(E + ident) * 0.01)
    x = rn(T, W)
    h = x.to(dtype)
    logits = x @ mlp.router.weight.data.T
    s = torch.softmax(logits[:, :E + ident], -1)
    choice = s + mlp.router.correction.data
    keep = choice.view(T, 4, -1).amax(-1).topk(2)[1]
    mask = torch.zeros(T, 4, dtype=torch.bool, device=DEV).scatter(1, keep, True).repeat_interleave((E + ident) // 4, 1)
    ids = choice.masked_fill(~mask, float("-inf")).topk(top)[1]
    wts = torch.zeros_like(s).scatter(1, ids, s.gather(1, ids))
    f = lambda z, up, down: torch.relu(z @ up.float().T) ** 2 @ down.float().T
    y = torch.sigmoid(logits[:, -1:]) * f(h.float(), mlp.shared.up.data, mlp.shared.down.data) + wts[:, E:].sum(-1, keepdim=True) * x
    for e in range(E):
        y += wts[:, e:e + 1] * f(h.float(), mlp.experts.up.data[e], mlp.experts.down.data[e])
    want = rms(3.0 * x + y, 1e-5)
    lo = norm(x, mlp(h, x), dtype)
    close(x, want, bar)
    close(lo, want, bar)
