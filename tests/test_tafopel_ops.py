"""Every mechanism the Tafopel family added to the operators, alone, against the plain restatement in
tests/oracle_tafopel.py: on the CPU the engine's plumbing operators, on the GPU (marked gpu) the HIP kernels of libhymix
and libseqmix in float32 and bfloat16.  Batches are built by hand: several sequences, portions that start in the middle
of a sequence, scattered cache blocks and state slots that hold stale data."""
import math
import os
import sys

import pytest
import torch

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, os.path.join(ROOT, "nano-vllm-hw3_amd"))
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import oracle_tafopel as O  # noqa: E402
from test_hymix_ops import CASES, F64, batch, gen, near, rnd  # noqa: E402  (operator test helpers)
from test_lilevik_ops import module, run_cut, stale  # noqa: E402

from nanovllm import hy_ops, seq_ops  # noqa: E402
from nanovllm.layers.f32_product import F32Product  # noqa: E402
from nanovllm.layers.feedforward import GatedMLP, ReluSquaredMLP, RoutedExperts  # noqa: E402
from nanovllm.layers.latent_attention import LatentAttention  # noqa: E402
from nanovllm.layers.parallel_block import ParallelBlock  # noqa: E402
from nanovllm.layers.selective_scan import SelectiveScan  # noqa: E402

CUTS = [[61, 3, 1, 64, 1, 1, 19], [70], [2, 1, 1, 5]]
LENGTHS = [150, 70, 9]


# ------------------------------------------------------------------------------------------ residual side
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W", [40, 7, 264, 1028, 2600, 4100])
def test_layer_norm_residual(device, dtype, W):
    """All forms: the embedding, one and two results, a token's expert rows with and without weights; a mean far from
    zero, which a variance taken as a difference of large sums would lose."""
    g = gen(W)
    T, eps, top = 9, 1e-5, 3
    embed = rnd(g, 19, W, dtype=dtype)
    ids = torch.randint(0, 19, (T,), generator=g)
    w1, w2 = 1 + rnd(g, W, s=0.2, dtype=dtype), 1 + rnd(g, W, s=0.2, dtype=dtype)
    norm = lambda z, w: O.layer_norm(z, w.to(F64), eps)  # noqa: E731
    x, h = hy_ops.layer_norm_residual(None, embed.to(device), w1.to(device), eps, dtype, ids=ids.to(device))
    ref = embed[ids].to(F64)
    near(x, ref, torch.float32, f32=1e-6)
    near(h, norm(ref, w1), dtype)
    assert x.dtype == torch.float32 and h.dtype == dtype
    y, y2 = 50 + rnd(g, T, W, s=3.0, dtype=dtype), rnd(g, T, W, dtype=dtype)
    x, h = hy_ops.layer_norm_residual(x, y.to(dtype).to(device), w2.to(device), eps, dtype, y2=y2.to(device))
    ref = ref + y.to(dtype).to(F64) + y2.to(F64)
    near(x, ref, torch.float32, f32=1e-6)
    near(h, norm(ref, w2), dtype, f32=5e-5)
    x, h = hy_ops.layer_norm_residual(x, y2.to(device), None, eps, dtype, routed=(y2.to(device), None, None))
    ref = ref + 2 * y2.to(F64)
    near(x, ref, torch.float32, f32=1e-6)
    assert h is None
    if device == "cuda":
        prod = rnd(g, 40, W, dtype=dtype)
        rows = torch.randint(0, 40, (T * top,), generator=g).int()
        for wts in (None, torch.rand(T, top, generator=g)):
            x, h = hy_ops.layer_norm_residual(x, y2.to(device), w1.to(device), eps, dtype,
                                              routed=(prod.to(device), rows.to(device), wts.to(device) if wts is not None else None))
            p = prod[rows.long()].to(F64).view(T, top, W)
            ref = ref + y2.to(F64) + ((p if wts is None else p * wts.to(F64)[..., None]).sum(1))
            near(x, ref, torch.float32, f32=1e-6)
            near(h, norm(ref, w1), dtype, f32=5e-5)


# ------------------------------------------------------------------------------------------ short convolution
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("C,taps", [(40, 4), (7, 2), (64, 1), (1100, 3), (24, 5), (16, 16), (128, 4)])
def test_short_conv_with_bias_and_silu(device, dtype, C, taps):
    """Portions of unequal sizes, down to single tokens shorter than the taps; x is a column slice of a wider product; the
    slots start full of another sequence's values."""
    g = gen(C + taps)
    w, b = rnd(g, C, taps, s=0.6, dtype=dtype), rnd(g, C, s=0.5, dtype=dtype)
    hs = [rnd(g, n, 2 * C, dtype=dtype) for n in LENGTHS]
    refs = [O.silu(O.causal_conv(h[:, C:].to(F64), w.to(F64), b.to(F64))) for h in hs]
    st = {}

    def caches(blocks, slots):
        st["s"] = torch.empty(slots, 1, max(taps - 1, 1), C, dtype=dtype, device=device)
        stale(st["s"], g)
    outs = run_cut(None, hs, CUTS, device, dtype, C, caches, forward=lambda x: seq_ops.short_conv(
        x[:, C:], w.to(device), st["s"], 0, seq_ops.get_step(), b.to(device), silu=True))
    for o, r in zip(outs, refs):
        near(o, r, dtype)


# ------------------------------------------------------------------------------------------ selective scan
SCAN_SIZES = [(40, 16), (7, 8), (33, 5), (130, 1), (24, 32), (12, 33), (20, 64), (9, 100), (6, 200), (5, 512), (300, 16)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("C,N", SCAN_SIZES)
def test_selective_scan_operator(device, dtype, C, N):
    """The recurrence alone, state counts on and off the register tiles; step sizes from tiny to large (softplus of -12 to
    12), decays from none to immediate."""
    g = gen(C * 3 + N)
    bias, D = rnd(g, C), 1 + rnd(g, C, s=0.3)
    A = -torch.exp(rnd(g, C, N, s=1.5))
    hs = []
    for n in LENGTHS:
        hs.append(torch.cat([rnd(g, n, C, dtype=dtype), rnd(g, n, 2 * N, dtype=dtype), rnd(g, n, C, s=2.0, dtype=dtype)], 1))
    pre = [rnd(g, n, C, s=4.0) for n in LENGTHS]
    refs = []
    for h, d in zip(hs, pre):
        h = h.to(F64)
        y, _ = O.selective_scan(h[:, :C], O.softplus(d.to(F64) + bias.to(F64)), A.to(F64), h[:, C:C + N], h[:, C + N:C + 2 * N], D.to(F64))
        refs.append(y * O.silu(h[:, C + 2 * N:]))
    st = {}

    def caches(blocks, slots):
        st["s"] = torch.empty(slots, C, N, device=device)
        stale(st["s"], g)
    both = [torch.cat([h.float(), d], 1) for h, d in zip(hs, pre)]       # (carried in float32: the values are the storage type's)

    def step(x):
        h, d = x[:, :2 * C + 2 * N].to(dtype), x[:, 2 * C + 2 * N:]
        out = torch.empty(x.shape[0], C + 3, dtype=dtype, device=device)
        hy_ops.selective_scan(h[:, :C], d, bias.to(device), h, C, C + N, A.to(device), D.to(device), h[:, C + 2 * N:], st["s"],
                              seq_ops.get_step(), out=out[:, 3:])
        return out[:, 3:]
    outs = run_cut(None, both, CUTS, device, dtype, C, caches, forward=step)
    for o, r in zip(outs, refs):
        near(o, r, dtype, f32=5e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("N", [8, 16, 24, 64, 128])
def test_selective_scan_forms_agree(N):
    """Large and small batches of the same sequence take different numbers of states per lane; each gives the same result."""
    g = gen(N)
    C, n = 512, 40
    x, z, bc, d = (rnd(g, n, k, dtype=torch.float32).cuda() for k in (C, C, 2 * N, C))
    A, bias, D = -torch.exp(rnd(g, C, N)).cuda(), rnd(g, C).cuda(), rnd(g, C).cuda()
    outs = []
    for B in (1, 6, 20, 200):
        ctx, _ = batch([(0, n)] * B, device="cuda", seed=B)
        state = torch.zeros(B + 2, C, N, device="cuda")
        rep = lambda t: t.repeat(B, 1)  # noqa: E731
        y = hy_ops.selective_scan(rep(x), rep(d), bias, rep(bc), 0, N, A, D, rep(z), state, ctx)
        assert torch.equal(y[:n], y[-n:])
        outs.append(y[:n])
    for o in outs[1:]:
        near(o, outs[0].cpu(), torch.float32, f32=1e-5)


def scan_layer(device, dtype, W, C, N, taps, R, g):
    mod = module(dtype, lambda: SelectiveScan(W, C, N, taps, R))
    p = {"mix.in": rnd(g, 2 * C, W, s=2 * W ** -0.5, dtype=dtype), "mix.conv": rnd(g, C, taps, s=0.6, dtype=dtype),
         "mix.conv.b": rnd(g, C, s=0.3, dtype=dtype), "mix.x": rnd(g, R + 2 * N, C, s=2 * C ** -0.5, dtype=dtype),
         "mix.dt": rnd(g, C, R, s=R ** -0.5, dtype=dtype), "mix.dt.b": rnd(g, C, dtype=torch.bfloat16) - 1,
         "mix.A_log": rnd(g, C, N, dtype=torch.bfloat16), "mix.D": 1 + rnd(g, C, s=0.2, dtype=torch.bfloat16),
         "mix.o": rnd(g, W, C, s=C ** -0.5, dtype=dtype)}
    for name, par in (("mix.in", mod.in_proj), ("mix.conv", mod.conv.weight), ("mix.conv.b", mod.conv.bias), ("mix.x", mod.x_proj),
                      ("mix.dt", mod.dt_proj), ("mix.dt.b", mod.dt_bias), ("mix.D", mod.D), ("mix.o", mod.o_proj)):
        par.data.copy_(p[name])
    mod.A.data.copy_(-torch.exp(p["mix.A_log"].float()))
    return mod.to(device), p, dict(inner=C, state=N, conv=taps, dt_rank=R)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W,C,N,taps,R", [(32, 48, 16, 4, 3), (24, 40, 8, 2, 8), (16, 20, 24, 3, 1), (40, 136, 16, 4, 24), (32, 64, 4, 1, 16),
                                          (64, 264, 16, 4, 200)])
def test_selective_scan_layer(device, dtype, W, C, N, taps, R):
    g = gen(W + C)
    mod, p, m = scan_layer(device, dtype, W, C, N, taps, R, g)
    hs = [rnd(g, n, W, dtype=dtype) for n in LENGTHS]
    p64 = {k: v.to(F64) for k, v in p.items()}
    refs = [O.mamba_mixer(h.to(F64), p64, m) for h in hs]

    def caches(blocks, slots):
        mod.allocate(slots, dtype, device)
        stale(mod.state, g)                    # a slot is never cleared: a portion at position 0 starts from zero by position
        stale(mod.conv.state, g)
    outs = run_cut(mod, hs, CUTS, device, dtype, C, caches)
    for o, r in zip(outs, refs):
        near(o, r, dtype, f32=5e-5, bf16=4e-2)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("sizes", [[1], [2], [7], [17], [500]])
def test_selective_scan_long_memory(device, dtype, sizes):
    """500 tokens in portions of several sizes and at once, with channels that hardly forget (A close to 0): what the first
    tokens left is still most of the state at the end, and it has travelled through the slot between all steps."""
    g = gen(3)
    mod, p, m = scan_layer(device, dtype, 16, 24, 8, 4, 4, g)
    p["mix.A_log"] = torch.full_like(p["mix.A_log"], -10.0)
    mod.A.data.copy_(-torch.exp(p["mix.A_log"].float()))
    n = 500
    hs = [rnd(g, n, 16, dtype=dtype)]
    p64 = {k: v.to(F64) for k, v in p.items()}
    ref = O.mamba_mixer(hs[0].to(F64), p64, m)
    late = O.mamba_mixer(hs[0][100:].to(F64), p64, m)
    assert (ref[-50:] - late[-50:]).abs().max() > 0.2 * ref[-50:].abs().max()       # the first tokens matter at the end

    def caches(blocks, slots):
        mod.allocate(slots, dtype, device)
        stale(mod.state, g)
        stale(mod.conv.state, g)
    cuts = [[sizes[0]] * (n // sizes[0]) + ([n % sizes[0]] if n % sizes[0] else [])]
    near(run_cut(mod, hs, cuts, device, dtype, 5, caches)[0], ref, dtype, f32=5e-5, bf16=4e-2)


@pytest.mark.parametrize("device,dtype", CASES)
def test_f32_product(device, dtype):
    g = gen(2)
    for T, K, N in ((5, 24, 40), (70, 3, 9), (1, 128, 64)):
        x, w = rnd(g, T, K + 5, dtype=dtype), rnd(g, N, K, dtype=dtype)
        y = F32Product()(x.to(device)[:, 2:2 + K], w.to(device))
        assert y.dtype == torch.float32
        near(y, x[:, 2:2 + K].to(F64) @ w.to(F64).T, torch.float32, f32=1e-5)


# ------------------------------------------------------------------------------------------ latent attention
def latent_layer(device, dtype, W, m, g, source=None, sink_shift=0.0):
    H, D, Rd, V, R, Q = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
    mod = module(dtype, lambda: LatentAttention(W, H, D, V, R, m["scale"], 1e-5, rot_dim=Rd, rot_dims=Rd, rot_base=m["rot"]["base"], q_rank=Q,
                                                rot_scaling=m["rot"].get("scaling"), sink=True, kv_source=source))
    p = {"mix.dq": rnd(g, Q, W, s=2 * W ** -0.5, dtype=dtype), "mix.dq.norm": 1 + rnd(g, Q, s=0.2, dtype=dtype),
         "mix.uq": rnd(g, H * (D + Rd), Q, s=2 * Q ** -0.5, dtype=dtype), "mix.uk": rnd(g, H * D, R, s=R ** -0.5, dtype=dtype),
         "mix.uv": rnd(g, H * V, R, s=R ** -0.5, dtype=dtype), "mix.o": rnd(g, W, H * V, s=(H * V) ** -0.5, dtype=dtype),
         "mix.sink": sink_shift + rnd(g, H, s=2.0, dtype=torch.bfloat16)}
    firsts = [p["mix.dq"]]
    if source is None:
        p.update({"mix.dkv": rnd(g, R + Rd, W, s=2 * W ** -0.5, dtype=dtype), "mix.dkv.norm": 1 + rnd(g, R, s=0.2, dtype=dtype)})
        firsts.append(p["mix.dkv"])
        mod.latent_norm.data.copy_(p["mix.dkv.norm"])
    mod.qc_proj.data.copy_(torch.cat(firsts))
    mod.q_latent_norm.data.copy_(p["mix.dq.norm"])
    mod.uq.data.copy_(p["mix.uq"])
    mod.uk.data.copy_(p["mix.uk"].view(H, D, R))
    mod.uv.data.copy_(p["mix.uv"].view(H, V, R).transpose(1, 2))
    mod.o_proj.data.copy_(p["mix.o"])
    mod.sink.data.copy_(p["mix.sink"].float())
    return mod.to(device), p


def latent_sizes(H=3, D=8, Rd=8, V=16, R=24, Q=20, scale=0.3, base=50.0, scaling=dict(factor=4.0, original=64, fast=8.0, slow=1.0)):
    rot = dict(dims=Rd, base=base)
    if scaling:
        rot["scaling"] = scaling
    return dict(heads=H, dim=D, rot_dim=Rd, vdim=V, kv_rank=R, q_rank=Q, scale=scale, rot=rot)


LATENT = [latent_sizes(), latent_sizes(1, 4, 2, 4, 8, 4, scaling=dict(factor=2.0, original=16, fast=4.0, slow=0.5)),
          latent_sizes(2, 40, 24, 72, 136, 56, base=10000.0), latent_sizes(4, 24, 8, 40, 112, 64, scaling=None),
          latent_sizes(5, 16, 12, 8, 41, 12), latent_sizes(40, 8, 16, 8, 48, 24), latent_sizes(2, 16, 64, 16, 192, 16),
          latent_sizes(130, 4, 8, 4, 24, 8)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("m", LATENT, ids=lambda m: f"H{m['heads']}R{m['kv_rank']}+{m['rot_dim']}")
def test_latent_attention_with_sink_stretched_rotation_and_a_reader(device, dtype, m):
    """A layer and a second one that reads its cached rows with queries and up-projections of its own, in the order the engine
    runs them: whole prompts, portions, single tokens, three sequences per step over stale pages."""
    g = gen(m["heads"] + m["kv_rank"])
    W = 32
    first, p = latent_layer(device, dtype, W, m, g)
    m2 = dict(m, heads=m["heads"] + 1, dim=m["dim"] + 4, vdim=m["vdim"] * 2, q_rank=m["q_rank"] + 4, scale=m["scale"] * 0.8)
    second, p2 = latent_layer(device, dtype, W, m2, g, source=first)
    assert second.cache_bytes_per_token(2) == 0 and second.qc_proj.shape[0] == m2["q_rank"]
    hs = [rnd(g, n, 2 * W, dtype=dtype) for n in LENGTHS]                # each layer reads an input of its own
    p64, q64 = {k: v.to(F64) for k, v in p.items()}, {k: v.to(F64) for k, v in p2.items()}
    refs = []
    for h in hs:
        a, b = h[:, :W].to(F64), h[:, W:].to(F64)
        rows = O.latent_rows(a, p64, m, 1e-5)
        kept = [r.to(dtype).to(F64) for r in rows]
        refs.append(torch.cat([O.latent_attention(a, *kept, p64, m, 1e-5), O.latent_attention(b, *kept, q64, m2, 1e-5)], 1))

    def caches(blocks, slots):
        first.allocate(0, blocks, 64, dtype, device)
        second.allocate(0, blocks, 64, dtype, device)
        assert second.cache[0] is first.cache[0]
        stale(first.cache[0], g)

    def step(x):
        a = first(x[:, :W].contiguous())
        return torch.cat([a, second(x[:, W:].contiguous())], 1)
    outs = run_cut(None, hs, CUTS, device, dtype, m["heads"], caches, forward=step)
    for o, r in zip(outs, refs):
        near(o[:, :W], r[:, :W], dtype, f32=5e-5, bf16=4e-2)
        near(o[:, W:], r[:, W:], dtype, f32=5e-5, bf16=4e-2)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("force_rows", [False, True])
@pytest.mark.parametrize("sink", [None, -30.0, 0.0, 3.0, 12.0, 60.0])
def test_sink_in_attention_alone(device, dtype, force_rows, sink):
    """Sinks from far below the scores to far above them (the output then goes to zero smoothly, with no overflow), on the
    matrix-core and the portable kernels, in prompts and in decoding; one key at the first position, at a page's borders and
    far back stands out for chosen queries."""
    g = gen(7)
    H, R, RV, n, scale = 3, 40, 32, 300, 0.25
    keys = rnd(g, n, R, s=0.5, dtype=dtype)
    q = rnd(g, n, H, R, s=0.5, dtype=dtype)
    for at, back in ((290, 0), (291, 63), (292, 64), (293, 127), (294, 128), (295, 200), (64, 0), (63, 1), (5, 5), (299, 299)):
        v = rnd(g, R, dtype=dtype)
        keys[back] = (v * 3).to(dtype)
        q[at] = (v * 2).to(dtype)
    s_vec = None if sink is None else sink + torch.tensor([0.0, 0.7, -1.1])
    s = torch.einsum("ihr,jr->hij", q.to(F64), keys.to(F64)) * scale
    i = torch.arange(n)
    s = s.masked_fill(i[:, None] < i[None, :], float("-inf"))
    w = torch.softmax(s, -1) if sink is None else O.sink_softmax(s, s_vec.to(F64)[:, None, None])
    ref = torch.einsum("hij,jv->ihv", w, keys[:, :RV].to(F64))
    dev_sink = None if sink is None else s_vec.to(device)
    for portions in ([(0, n)], [(250, n - 250)], [(n - 1, 1)], [(64, 1)], [(0, 1)]):
        ctx, blocks = batch(portions, device=device, seed=11)
        cache = torch.empty(blocks, 64, R, dtype=dtype, device=device)
        stale(cache, g)
        p0, m = portions[0]
        bt = ctx.block_tables[0].cpu().tolist()
        rows = torch.tensor([bt[j // 64] * 64 + j % 64 for j in range(p0 + m)])
        cache.view(-1, R)[rows.to(device)] = keys[:p0 + m].to(device)
        o = seq_ops.latent_attention(q[p0:p0 + m].to(device).contiguous(), cache, ctx, scale, force_rows=force_rows, value_cols=RV, sink=dev_sink)
        want = ref[p0:p0 + m]
        got = o.detach().cpu().to(F64)
        assert torch.isfinite(got).all()
        assert (got - want).abs().max() < (3e-5 if dtype == torch.float32 else 2e-2) * max(want.abs().max().item(), 1e-3)


def test_stretched_table_of_a_latent_layer():
    """The layer's table and factor are the oracle's, for tables stretched over all, some and none of their pairs; a
    reader's rotation is its source's."""
    for rot in (dict(dims=8, base=100.0, scaling=dict(factor=4.0, original=64, fast=8.0, slow=1.0)), dict(dims=24, base=10000.0),
                dict(dims=64, base=500000.0, scaling=dict(factor=32.0, original=4096, fast=32.0, slow=1.0)),
                dict(dims=2, base=10.0, scaling=dict(factor=2.0, original=16, fast=4.0, slow=0.5))):
        mod = module(torch.float32, lambda: LatentAttention(8, 1, 4, 4, 8, 1.0, 1e-5, rot_dim=rot["dims"], rot_dims=rot["dims"],
                                                            rot_base=rot["base"], q_rank=4, rot_scaling=rot.get("scaling"), sink=True))
        mod.allocate(0, 1, 64, torch.float32, "cpu")
        f, mag = O.rotary_table(rot)
        assert torch.allclose(mod.inv_freq.double(), f, rtol=1e-6, atol=0) and abs(mod.rot_mag - mag) < 1e-12
        sc = rot.get("scaling")
        assert mod.rot_mag == (0.1 * math.log(sc["factor"]) + 1.0 if sc else 1.0)


# ------------------------------------------------------------------------------------------ feed-forward
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W,ff,T", [(32, 40, 9), (24, 7, 5), (64, 128, 70)])
def test_gated_mlp(device, dtype, W, ff, T):
    g = gen(ff)
    mod = module(dtype, lambda: GatedMLP(W, ff, "gelu_tanh_glu"))
    p = {"mlp.gate": rnd(g, ff, W, s=3 * W ** -0.5, dtype=dtype), "mlp.up": rnd(g, ff, W, s=2 * W ** -0.5, dtype=dtype),
         "mlp.down": rnd(g, W, ff, s=ff ** -0.5, dtype=dtype)}
    mod.gate_up.data.copy_(torch.cat([p["mlp.gate"], p["mlp.up"]]))
    mod.down.data.copy_(p["mlp.down"])
    h = rnd(g, T, W, dtype=dtype)
    near(mod.to(device)(h.to(device)), O.dense(h.to(F64), {k: v.to(F64) for k, v in p.items()}), dtype, f32=3e-5, bf16=4e-2)


def moe_layer(device, dtype, W, E, top, ff, fs, g):
    mod = module(dtype, lambda: RoutedExperts(W, E, top, ff, shared=ReluSquaredMLP(W, fs) if fs else None, score="sigmoid", renorm=False,
                                              act="relu_sq", weight_in=True, shared_gate=bool(fs)))
    p = {"mlp.router": rnd(g, E, W, s=3 * W ** -0.5, dtype=torch.bfloat16)}
    for e in range(E):
        p.update({f"mlp.e{e}.up": rnd(g, ff, W, s=2 * W ** -0.5, dtype=dtype), f"mlp.e{e}.down": rnd(g, W, ff, s=ff ** -0.5, dtype=dtype)})
        mod.w_gu.data[e].copy_(p[f"mlp.e{e}.up"])
        mod.w_down.data[e].copy_(p[f"mlp.e{e}.down"])
    mod.router.data.copy_(p["mlp.router"].float())
    if fs:
        p.update({"mlp.shared.up": rnd(g, fs, W, s=2 * W ** -0.5, dtype=dtype), "mlp.shared.down": rnd(g, W, fs, s=fs ** -0.5, dtype=dtype),
                  "mlp.shared.sg": rnd(g, 1, W, s=3 * W ** -0.5, dtype=torch.bfloat16)})
        mod.shared.up.data.copy_(p["mlp.shared.up"])
        mod.shared.down.data.copy_(p["mlp.shared.down"])
        mod.shared_gate.data.copy_(p["mlp.shared.sg"].float().view(-1))
    cfg = dict(kind="moe", router=dict(experts=E, top=top), expert=dict(ff=ff), shared=dict(ff=fs) if fs else None)
    return mod.to(device), p, cfg


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W,E,top,ff,fs,T", [(32, 8, 3, 24, 40, 19), (48, 6, 2, 16, 0, 1), (64, 4, 4, 40, 24, 300), (40, 5, 1, 8, 8, 64),
                                             (20, 3, 2, 7, 5, 33), (24, 1, 1, 16, 16, 10), (264, 12, 5, 72, 16, 40)])
def test_experts_weighted_at_their_input_and_gated_shared_expert(device, dtype, W, E, top, ff, fs, T):
    """The whole feed-forward against the oracle, on the GPU in bfloat16 in all three forms; then its parts: routed rows left
    to the residual boundary, the shared expert scaled before its last product.  Squared ReLU of a scaled input is the
    square of the weight on the output: a weight applied to the output once instead would show."""
    g = gen(W + T)
    mod, p, cfg = moe_layer(device, dtype, W, E, top, ff, fs, g)
    p64 = {k: v.to(F64) for k, v in p.items()}
    h = rnd(g, T, W, dtype=dtype)
    ref = O.mixture(h.to(F64), p64, cfg)
    dh = h.to(device)
    near(mod(dh), ref, dtype, f32=3e-5, bf16=4e-2)
    idx, wts, gate = mod.route(dh)
    ridx, rwts = O.route(h.to(F64), p64["mlp.router"], top)
    order, rorder = idx.cpu().long().sort(-1), ridx.sort(-1)
    assert torch.equal(order.values, rorder.values)
    near(wts.cpu().gather(1, order.indices), rwts.gather(1, rorder.indices), torch.float32, f32=2e-5)
    wrong = torch.zeros_like(ref)                                       # the weight on the output instead
    for t in range(T):
        for e, w in zip(ridx[t].tolist(), rwts[t]):
            wrong[t] += w * O.expert(h[t].to(F64), p64, f"mlp.e{e}")
    routed = ref if not fs else ref - torch.sigmoid(h.to(F64) @ p64["mlp.shared.sg"].T) * O.expert(h.to(F64), p64, "mlp.shared")
    assert (wrong - routed).abs().max() > 0.05 * routed.abs().max()
    if fs:
        near(gate, torch.sigmoid(h.to(F64) @ p64["mlp.shared.sg"].T)[:, 0], torch.float32, f32=2e-5)
    x = torch.zeros(T, W, device=device)
    rows = mod.products(dh, idx, wts, combine=False)
    x, _ = hy_ops.layer_norm_residual(x, torch.zeros(T, W, dtype=dtype, device=device), None, 1e-5, dtype, routed=rows)
    near(x, routed, dtype, f32=3e-5, bf16=4e-2)
    if device == "cuda" and dtype == torch.bfloat16 and W % 8 == 0 and ff % 8 == 0:
        for form in ("pairs", "grouped", "tiles128"):
            kw = dict(form=form, act_kind=seq_ops.ACT_RELU_SQ, weight_in=True)
            shared = mod.shared(dh)[0] if fs else None
            y = seq_ops.moe_experts(dh, idx, wts, mod.w_gu, mod.w_down, 0.0, 1.0, shared, shared_scale=gate, **kw)
            near(y, ref, dtype, bf16=4e-2)
            if form != "pairs":
                left = seq_ops.moe_experts(dh, idx, wts, mod.w_gu, mod.w_down, 0.0, 1.0, combine=False, **kw)
                assert left[1] is not None and left[2] is None


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("T", [1, 37, 1501, 4103])
@pytest.mark.parametrize("W,E,top,score,groups", [(64, 16, 4, "sigmoid", 1), (40, 70, 8, "softmax", 1), (30, 5, 5, "sigmoid", 1), (16, 200, 32, "softmax", 1),
                                                  (24, 300, 3, "sigmoid", 1), (48, 12, 3, "softmax", 4)])
def test_router_step_sizes_and_scores(device, dtype, T, W, E, top, score, groups):
    """Steps of one token to thousands (the kernel takes different numbers of tokens per workgroup), more experts than lanes,
    both scores, with and without groups, biases, corrections that steer the choice, renormalised and plain weights."""
    g = gen(T + E)
    h = rnd(g, T, W, dtype=dtype)
    rw, bias, corr, gw = rnd(g, E, W, s=2 * W ** -0.5), rnd(g, E, s=0.3), rnd(g, E, s=0.2), rnd(g, W, s=W ** -0.5)
    z = h.to(F64) @ rw.to(F64).T + bias.to(F64)
    s = torch.sigmoid(z) if score == "sigmoid" else torch.softmax(z, -1)
    c = s + corr.to(F64)
    if groups > 1:
        best = c.view(T, groups, -1).max(-1).values.topk(2, -1).indices
        keep = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best, True)
        c = c.masked_fill(~keep.repeat_interleave(E // groups, 1), float("-inf"))
    for renorm in (False, True):
        idx, wts, gate = seq_ops.moe_route(h.to(device), rw.to(device), top, groups, 2 if groups > 1 else 1,
                                           seq_ops.ROUTE_SIGMOID if score == "sigmoid" else seq_ops.ROUTE_SOFTMAX, corr.to(device), 1, renorm,
                                           bias.to(device), gw.to(device))
        idx, wts = idx.cpu().long(), wts.cpu().to(F64)
        assert all(len(set(r)) == top for r in idx[:50].tolist())
        chosen = c.gather(1, idx)                          # (near-ties may fall either way: the choice scores decide)
        near(chosen.sort(-1).values, c.topk(top, -1).values.sort(-1).values, torch.float32, f32=2e-5)
        w = s.gather(1, idx)
        near(wts, w / w.sum(-1, keepdim=True) if renorm else w, torch.float32, f32=5e-5)
        near(gate, torch.sigmoid(h.to(F64) @ gw.to(F64)), torch.float32, f32=2e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("act", ["gelu", "clamped_glu", "silu_glu", "gelu_tanh_glu", "relu_sq"])
def test_input_weights_with_other_activations(dtype, act):
    """Weights on the experts' inputs under every activation, in every form, against the plain-torch counterpart."""
    from nanovllm import cpu_ops
    g = gen(len(act))
    W, E, top, ff, T = 48, 5, 2, 24, 50
    kind = RoutedExperts.ACTS[act]
    parts = 2 if kind in seq_ops.GATED_ACTS else 1
    h, w_gu, w_down = rnd(g, T, W, dtype=dtype), rnd(g, E, parts * ff, W, s=0.3, dtype=dtype), rnd(g, E, W, ff, s=0.2, dtype=dtype)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    wts = torch.rand(T, top, generator=g)
    limit, alpha = (1.5, 1.702) if act == "clamped_glu" else (float("inf"), 1.0)
    ref = cpu_ops.moe_experts(h.float(), idx, wts, w_gu.float(), w_down.float(), limit, alpha, None, kind, True)
    for form in ("pairs",) if dtype == torch.float32 else ("pairs", "grouped", "tiles128"):
        y = seq_ops.moe_experts(h.cuda(), idx.cuda(), wts.cuda(), w_gu.cuda(), w_down.cuda(), limit, alpha, form=form, act_kind=kind, weight_in=True)
        near(y, ref, dtype, f32=3e-5, bf16=4e-2)


# ------------------------------------------------------------------------------------------ parallel block
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", ["scan", "latent"])
@pytest.mark.parametrize("ff", ["none", "dense", "moe", "moe_alone"])
def test_parallel_block(device, dtype, kind, ff):
    """Mixer and feed-forward on one input: the merged products give what the two modules give, whatever rides on them."""
    g = gen(len(kind) + len(ff))
    W = 40
    if kind == "scan":
        mixer, p, m = scan_layer(device, dtype, W, 56, 16, 4, 6, g)
        run = lambda h, q: O.mamba_mixer(h, q, m)  # noqa: E731
    else:
        m = latent_sizes(R=56)
        mixer, p = latent_layer(device, dtype, W, m, g)
        run = lambda h, q: O.latent_attention(h, *[r.to(dtype).to(F64) for r in O.latent_rows(h, q, m, 1e-5)], q, m, 1e-5)  # noqa: E731
    mlp, add = None, lambda h, q: 0.0  # noqa: E731
    if ff == "dense":
        mlp = module(dtype, lambda: GatedMLP(W, 24, "gelu_tanh_glu")).to(device)
        p.update({"mlp.gate": rnd(g, 24, W, s=0.4, dtype=dtype), "mlp.up": rnd(g, 24, W, s=0.4, dtype=dtype), "mlp.down": rnd(g, W, 24, s=0.2, dtype=dtype)})
        mlp.gate_up.data.copy_(torch.cat([p["mlp.gate"], p["mlp.up"]]))
        mlp.down.data.copy_(p["mlp.down"])
        add = O.dense
    elif ff != "none":
        mlp, pm, cfg = moe_layer(device, dtype, W, 6, 2, 24, 16 if ff == "moe" else 0, g)
        p.update(pm)
        add = lambda h, q: O.mixture(h, q, cfg)  # noqa: E731
    block = ParallelBlock(mixer, mlp)
    hs = [rnd(g, n, W, dtype=dtype) for n in LENGTHS]
    p64 = {k: v.to(F64) for k, v in p.items()}
    refs = [run(h.to(F64), p64) + add(h.to(F64), p64) for h in hs]

    def caches(blocks, slots):
        if kind == "scan":
            mixer.allocate(slots, dtype, device)
            stale(mixer.state, g)
            stale(mixer.conv.state, g)
        else:
            mixer.allocate(0, blocks, 64, dtype, device)
            stale(mixer.cache[0], g)

    def step(h):
        y, rows = block(h)
        return hy_ops.layer_norm_residual(torch.zeros(h.shape, device=device), y, None, 1e-5, dtype, routed=rows)[0]
    outs = run_cut(None, hs, CUTS, device, dtype, 3, caches, forward=step)
    for o, r in zip(outs, refs):
        near(o, r, dtype, f32=5e-5, bf16=4e-2)
