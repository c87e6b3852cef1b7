"""The Tafopel model family in the engine against the plain restatement in tests/oracle_tafopel.py.

Every test makes its own small configuration and random checkpoint.  ``device`` = "cpu" drives the engine's plumbing
operators (scheduler, block and slot pools, portion batching are the same code as on the GPU); "cuda" (marked gpu) drives
the HIP kernels of libhymix and libseqmix, in float32 against tight bounds and in bfloat16 against the rounding of that
format."""
import os
import random
import sys

import numpy as np
import pytest
import torch

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, os.path.join(ROOT, "nano-vllm-hw3_amd"))
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import oracle_tafopel as O  # noqa: E402
from test_lilevik import close  # noqa: E402
from test_pasizen import DEVICES, cut, dtypes_for, replay, tokens, write_model  # noqa: E402  (engine test helpers)


def scan(inner=56, state=16, conv=4, dt_rank=6):
    return "mamba1", dict(inner=inner, state=state, conv=conv, dt_rank=dt_rank)


def latent(heads=3, dim=8, rot_dim=8, vdim=16, kv_rank=24, q_rank=20, scale=0.3, base=100.0, scaling=(4.0, 64, 8.0, 1.0), kv_from=None):
    rot = dict(dims=rot_dim, base=base)
    if scaling:
        rot["scaling"] = dict(factor=scaling[0], original=scaling[1], fast=scaling[2], slow=scaling[3])
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale, rot=rot)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "latent_attention", m


def dense(ff=40):
    return dict(kind="dense", ff=ff)


def moe(experts=8, top=3, ff=24, shared=16):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top), shared=dict(ff=shared) if shared else None)


def config(layers, width=48, vocab=61, eps=1e-5):
    return dict(architecture="Tafopel", vocab=vocab, width=width, norm=dict(eps=eps),
                layers=[dict(type=kind, mixer=m, mlp=mlp) for (kind, m), mlp in layers])


DEFAULT = [(latent(), moe()), (scan(), dense()), (latent(heads=2, dim=12, vdim=8, q_rank=8, scale=0.4, kv_from=0), None),
           (scan(inner=40, state=8, conv=3, dt_rank=2), moe(experts=6, top=2, ff=16, shared=24)),
           (latent(heads=4, rot_dim=4, kv_rank=40, scaling=None), dense(24)),
           (latent(heads=5, rot_dim=4, kv_rank=40, scaling=None, kv_from=4), moe(experts=4, top=1, shared=0)), (scan(state=24, conv=2), None)]


def weights(cfg, seed=0, sink=0.0):
    """A random checkpoint under the design's tensor names, bf16-representable values."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def rnd(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(torch.bfloat16)
    t = {"embed": rnd(cfg["vocab"], W, s=0.7), "final.norm": 1 + rnd(W, s=0.2), "head": rnd(cfg["vocab"], W, s=W ** -0.5)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        t[p + "norm1"] = 1 + rnd(W, s=0.2)
        if L["type"] == "mamba1":
            C, N, K, R = m["inner"], m["state"], m["conv"], m["dt_rank"]
            t.update({p + "mix.in": rnd(2 * C, W, s=W ** -0.5), p + "mix.conv": rnd(C, K, s=K ** -0.5), p + "mix.conv.b": rnd(C, s=0.3),
                      p + "mix.x": rnd(R + 2 * N, C, s=1.5 * C ** -0.5), p + "mix.dt": rnd(C, R, s=R ** -0.5), p + "mix.dt.b": rnd(C) - 1.5,
                      p + "mix.A_log": rnd(C, N, s=1.0) - 0.5, p + "mix.D": 1 + rnd(C, s=0.2), p + "mix.o": rnd(W, C, s=C ** -0.5)})
        else:
            H, D, V, R, Rd, Q = m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["rot_dim"], m["q_rank"]
            t.update({p + "mix.dq": rnd(Q, W, s=2 * W ** -0.5), p + "mix.dq.norm": 1 + rnd(Q, s=0.2),
                      p + "mix.uq": rnd(H * (D + Rd), Q, s=2 * Q ** -0.5), p + "mix.uk": rnd(H * D, R, s=R ** -0.5),
                      p + "mix.uv": rnd(H * V, R, s=R ** -0.5), p + "mix.o": rnd(W, H * V, s=(H * V) ** -0.5), p + "mix.sink": sink + rnd(H)})
            if m.get("kv_from") is None:
                t.update({p + "mix.dkv": rnd(R + Rd, W, s=2 * W ** -0.5), p + "mix.dkv.norm": 1 + rnd(R, s=0.2)})
        mlp = L["mlp"]
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            ff = mlp["ff"]
            t.update({p + "mlp.gate": rnd(ff, W, s=2 * W ** -0.5), p + "mlp.up": rnd(ff, W, s=W ** -0.5), p + "mlp.down": rnd(W, ff, s=ff ** -0.5)})
            continue
        E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        t[p + "mlp.router"] = rnd(E, W, s=3 * W ** -0.5)
        for e in range(E):
            t.update({f"{p}mlp.e{e}.up": rnd(ff, W, s=1.5 * W ** -0.5), f"{p}mlp.e{e}.down": rnd(W, ff, s=ff ** -0.5)})
        if mlp["shared"]:
            fs = mlp["shared"]["ff"]
            t.update({p + "mlp.shared.up": rnd(fs, W, s=W ** -0.5), p + "mlp.shared.down": rnd(W, fs, s=fs ** -0.5),
                      p + "mlp.shared.sg": rnd(1, W, s=2 * W ** -0.5)})
    return {k: v.to(torch.bfloat16).contiguous() for k, v in t.items()}


# share of rows a turned near-tie of these small random routers may move in bfloat16: a token whose expert changed also
# stays in the scan layers' state and in the cache, so rows behind it move with it
BF16_TIES = 0.2


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = config(DEFAULT)
    w = weights(cfg, seed=1)
    return write_model(tmp_path_factory.mktemp("tafopel_default"), cfg, w), cfg, w


def forward(cfg, w, toks):
    return O.forward(cfg, w, toks)[0].numpy()


# ------------------------------------------------------------------------------------------ whole model, schedules
@pytest.mark.parametrize("device", DEVICES)
def test_whole_prompt_and_layer_trace(model, tmp_path, device):
    """One step per prompt: every position's logits; and the residual after every layer, through the runner itself."""
    path, cfg, w = model
    toks = tokens(90, cfg["vocab"], 3)
    ref, layers = O.forward(cfg, w, toks)
    for dtype in dtypes_for(device):
        got = replay(path, [([("a", toks, list(range(90)))], ["a"])], tmp_path, device, dtype)
        close(got[0], ref.numpy(), dtype, BF16_TIES)
    from nanovllm.engine.llm_engine import LLMEngine
    from nanovllm.engine.sequence import ACTIVE, Sequence
    eng = LLMEngine(path, device=device, dtype=torch.float32, max_num_seqs=2, num_kvcache_blocks=4, max_num_batched_tokens=4096)
    seq = Sequence(toks)
    seq.state = ACTIVE
    assert eng.scheduler.reserve_portion(seq, 90)
    trace = []
    eng.model_runner.run_portions([(seq, 90)], trace=trace)
    assert len(trace) == len(layers) == len(cfg["layers"])
    for got_l, ref_l in zip(trace, layers):
        assert torch.allclose(got_l.cpu().double(), ref_l, atol=3e-4, rtol=3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_prefill_equals_token_by_token(model, tmp_path, device):
    """A prompt fed one token per step (caches, states and convolution inputs built from the very first token) gives the
    logits of the whole prompt in one step; 150 tokens cross two cache-block borders."""
    path, cfg, w = model
    toks = tokens(150, cfg["vocab"], 4)
    ref = forward(cfg, w, toks)
    steps = [([("a", [t], [0])], ["a"] if i == 149 else []) for i, t in enumerate(toks)]
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=192)
        close(np.concatenate([got[i] for i in range(150)]), ref, dtype, BF16_TIES)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("sizes", [[2], [3, 2, 7, 2, 64, 1, 5], [63, 2, 1, 64], [65, 1, 1, 1, 2], [16, 17, 15, 2]])
def test_portions(model, tmp_path, device, sizes):
    """Prompts cut into portions of several sizes (down to two tokens, across cache-block borders and the kernels' token
    chunks, single tokens between): rows, states and convolution inputs travel from portion to portion."""
    path, cfg, w = model
    toks = tokens(133, cfg["vocab"], 5)
    ref = forward(cfg, w, toks)
    parts = cut(133, sizes)
    steps = [([("r", toks[a:b], list(range(b - a)))], ["r"] if b == 133 else []) for a, b in parts]
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=192)
        close(np.concatenate([got[i] for i in range(len(parts))]), ref, dtype, BF16_TIES)


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_batches_and_reused_pages_and_slots(model, tmp_path, device):
    """Unequal requests share steps (prompt portions beside single tokens), more requests than state slots and more tokens
    than cache blocks over the run: blocks and slots are freed and taken again, also by requests whose first tokens land in a
    slot that still holds another's state, and by one shorter than the convolutions.  Each request equals itself alone."""
    path, cfg, w = model
    V = cfg["vocab"]
    reqs = {f"q{i}": tokens(n, V, 10 + i) for i, n in enumerate([97, 5, 130, 66, 1, 71, 64, 2])}
    ref = {k: forward(cfg, w, v) for k, v in reqs.items()}
    plan = {"q0": cut(97, [40, 1, 1, 30, 1]), "q1": cut(5, [2, 1]), "q2": cut(130, [64, 3, 1]), "q3": cut(66, [66]),
            "q4": cut(1, [1]), "q5": cut(71, [7, 1]), "q6": cut(64, [62, 2]), "q7": cut(2, [1])}
    live, waiting, steps, rows = [], list(reqs), [], []
    cursor = {k: 0 for k in reqs}
    while live or waiting:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        entries, end = [], []
        for j, k in enumerate(list(live)):
            if len(live) > 1 and j == len(steps) % 5:                   # left out of this step, goes on later
                continue
            a, b = plan[k][cursor[k]]
            cursor[k] += 1
            entries.append((k, reqs[k][a:b], list(range(b - a))))
            rows.append((len(steps), k, a, b))
            if b == len(reqs[k]):
                end.append(k)
                live.remove(k)
        steps.append((entries, end))
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=7 * 64, max_live=3)
        at, all_got, all_ref = {}, [], []
        for s, k, a, b in rows:
            o = at.get(s, 0)
            all_got.append(got[s][o:o + b - a])
            all_ref.append(ref[k][a:b])
            at[s] = o + b - a
        close(np.concatenate(all_got), np.concatenate(all_ref), dtype, BF16_TIES)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(model, tmp_path, device):
    """A short prompt and 200 single-token steps: three block borders pass over decoded tokens."""
    path, cfg, w = model
    toks = tokens(215, cfg["vocab"], 6)
    ref = forward(cfg, w, toks)
    steps = [([("a", toks[:15], [14])], [])] + [([("a", [t], [0])], []) for t in toks[15:]]
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=256)
        close(np.concatenate([got[i] for i in range(len(steps))]), ref[14:], dtype, BF16_TIES)


VARIANTS = {
    # sizes that the default makes equal are unequal here and the other way round; values of 1
    "latent_only_one_head": config([(latent(heads=1, dim=4, rot_dim=2, vdim=4, kv_rank=8, q_rank=4, scaling=(2.0, 16, 4.0, 0.5)), None)], width=16),
    "scan_only_one_state_one_tap": config([(scan(inner=24, state=1, conv=1, dt_rank=1), dense(8))], width=24),
    "readers_in_a_row": config([(latent(), dense(16)), (latent(kv_from=0), None), (scan(state=4, conv=5), None), (latent(heads=6, kv_from=0), moe()),
                                (latent(dim=4, vdim=4, q_rank=6, kv_from=0), moe(top=8))]),
    "all_experts_and_one": config([(scan(inner=48, state=32, dt_rank=48), moe(experts=4, top=4, ff=40, shared=8)),
                                   (latent(vdim=8), moe(experts=1, top=1, ff=16, shared=32))], width=64, eps=1e-3),
    "off_the_tiles": config([(scan(inner=37, state=11, conv=3, dt_rank=5), moe(experts=5, top=2, ff=13, shared=7)),
                             (latent(heads=2, dim=5, rot_dim=6, vdim=7, kv_rank=17, q_rank=9), dense(11))], width=30, vocab=53),
    "big_heads": config([(latent(heads=2, dim=40, rot_dim=24, vdim=72, kv_rank=136, q_rank=56), None),
                         (scan(inner=136, state=64, conv=4, dt_rank=24), None), (latent(heads=34, rot_dim=64, kv_rank=192, q_rank=16), None)]),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(VARIANTS))
def test_other_shapes(tmp_path, device, name):
    """Other sizes, orders and constants: each mixer alone, one head, one state, one tap, several readers of one layer, all
    experts and a single one, with and without a shared expert, sizes off the matrix-core tiles.  Portions and a batch."""
    cfg = VARIANTS[name]
    w = weights(cfg, seed=7)
    path = write_model(tmp_path / "m", cfg, w)
    a, b = tokens(150, cfg["vocab"], 8), tokens(9, cfg["vocab"], 9)
    ra, rb = forward(cfg, w, a), forward(cfg, w, b)
    steps = [([("a", a[:31], list(range(31)))], []),
             ([("a", a[31:131], list(range(100))), ("b", b[:2], [0, 1])], []),
             ([("b", b[2:], list(range(7))), ("a", a[131:132], [0])], ["b"])] + \
            [([("a", [t], [0])], []) for t in a[132:]]
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=256)
        allg = np.concatenate([got[i] for i in range(len(steps))])
        allr = np.concatenate([ra[:31], ra[31:131], rb[:2], rb[2:], ra[131:132], ra[132:]])
        close(allg, allr, dtype, BF16_TIES)


def random_config(seed):
    """A configuration drawn from the design's whole space: 1-6 layers of either mixer in any order, readers of any earlier
    latent layer, sizes on and off the matrix-core tiles, stretched and plain frequency tables, any feed-forward or none."""
    r = random.Random(seed)
    width = r.choice([32, 48, 64, 96, 136])
    layers, sources = [], []
    for i in range(r.randint(1, 6)):
        mlp = r.choice([None, dense(r.choice([8, 16, 24, 44])), 1, 1])
        if mlp == 1:
            experts = r.randint(1, 12)
            mlp = moe(experts=experts, top=r.randint(1, min(experts, 5)), ff=r.choice([8, 16, 24, 40]), shared=r.choice([0, 8, 16, 36]))
        if r.random() < 0.5:
            layers.append((scan(inner=r.choice([16, 24, 40, 72, 130]), state=r.choice([1, 4, 8, 16, 20, 32, 64]), conv=r.choice([1, 2, 3, 4, 6]),
                                dt_rank=r.choice([1, 3, 8, 20])), mlp))
            continue
        heads, dim, vdim, q_rank = r.choice([1, 2, 3, 4, 8]), r.choice([4, 8, 16, 32]), r.choice([4, 8, 16, 32]), r.choice([4, 12, 32, 50])
        if sources and r.random() < 0.5:
            j = r.choice(sources)
            (_, m), _ = layers[j]
            layers.append((("latent_attention", dict(m, heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_from=j)), mlp))
            continue
        sources.append(i)
        scaling = (r.choice([1.0, 2.0, 16.0]), r.choice([16, 64, 256]), r.choice([4.0, 32.0]), r.choice([0.5, 1.0])) if r.random() < 0.7 else None
        layers.append((latent(heads, dim, r.choice([2, 4, 8, 16, 32]), vdim, r.choice([8, 16, 24, 64, 96, 36]), q_rank, 0.2,
                              r.choice([50.0, 10000.0]), scaling), mlp))
    return config(layers, width=width, vocab=r.choice([37, 64, 200]))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("seed", range(8))
def test_random_configurations(tmp_path, device, seed):
    """Configurations drawn at random, in float32 (the sharp comparison; bfloat16 is bounded per mechanism and on the
    fixed configurations): a prompt in two portions, a second request beside it, then single tokens."""
    cfg = random_config(seed)
    w = weights(cfg, seed=seed)
    path = write_model(tmp_path / "m", cfg, w)
    n = 150
    a, b = tokens(n, cfg["vocab"], seed), tokens(40, cfg["vocab"], seed + 100)
    ra, rb = forward(cfg, w, a), forward(cfg, w, b)
    c1 = 1 + (seed * 37) % (n - 40)
    steps = [([("a", a[:c1], list(range(c1)))], []),
             ([("a", a[c1:n - 20], list(range(n - 20 - c1))), ("b", b[:7], list(range(7)))], []),
             ([("b", b[7:], list(range(33))), ("a", a[n - 20:n - 19], [0])], ["b"])] + [([("a", [t], [0])], []) for t in a[n - 19:]]
    got = replay(path, steps, tmp_path, device, torch.float32, max_tokens=256)
    close(np.concatenate([got[i] for i in range(len(steps))]),
          np.concatenate([ra[:c1], ra[c1:n - 20], rb[:7], rb[7:], ra[n - 20:n - 19], ra[n - 19:]]), torch.float32)


@pytest.mark.parametrize("device", DEVICES)
def test_far_tokens_and_sinks_show(tmp_path, device):
    """A model whose far tokens decide: steep scores whose keys follow the queries (equal tokens attract, wherever they are),
    in a layer and in one that reads its rows.  The repeated token lies far back, at a cache-block border and among the
    sequence's first tokens; the queries are decoded alone and as a prompt's rows.  Without the sinks (planted in the oracle) a
    query with no equal token before it would spread its weight over all keys instead of keeping it to itself."""
    lat = latent(heads=2, dim=16, rot_dim=4, vdim=16, kv_rank=16, q_rank=16, scale=1.2)
    cfg = config([(lat, None), ((lat[0], dict(lat[1], kv_from=0)), None)], width=32)
    w = weights(cfg, seed=5, sink=10.0)
    for i in (0, 1):
        # k_h = c (the up-projection copies the latent) and q_h = the query's own latent: tokens whose latents agree score high
        w[f"l{i}.mix.uk"] = torch.eye(16).repeat(2, 1).to(torch.bfloat16)
        w[f"l{i}.mix.dq"] = w["l0.mix.dkv"][:16].clone()
        w[f"l{i}.mix.dq.norm"] = w["l0.mix.dkv.norm"].clone()
        uq = torch.zeros(2, 20, 16)
        uq[:, :16] = torch.eye(16)
        w[f"l{i}.mix.uq"] = uq.reshape(40, 16).to(torch.bfloat16)
    path = write_model(tmp_path / "m", cfg, w)
    toks = tokens(420, cfg["vocab"], 13)
    toks[390:] = [t % 30 for t in toks[390:]]
    toks[2:390] = [30 + t % (cfg["vocab"] - 30) if j not in (63, 64, 127, 250, 389) else t for j, t in enumerate(toks[2:390], 2)]
    for k, (back, at) in enumerate(((0, 400), (1, 401), (63, 402), (64, 403), (127, 404), (250, 405), (389, 406))):
        toks[back] = toks[at] = k                                       # one earlier token equal to the query's
    ref = forward(cfg, w, toks)
    cut_off = forward(cfg, w, toks[130:])          # without the far tokens the rows differ much
    assert np.abs(ref[400:405] - cut_off[270:275]).max() > 0.05 * ref.std()
    no_sink = {k: v.clone() - 1000 if k.endswith("sink") else v for k, v in w.items()}
    assert np.abs(ref[400:] - forward(cfg, no_sink, toks)[400:]).max() > 0.05 * ref.std()
    steps = [([("a", toks[:398], [397])], [])] + [([("a", [t], [0])], []) for t in toks[398:]]
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=448)
        close(np.concatenate([got[i] for i in range(len(steps))]), ref[397:], dtype)
        whole = replay(path, [([("a", toks[:200], []), ], []), ([("a", toks[200:], list(range(190, 220)))], ["a"])], tmp_path, device, dtype,
                       max_tokens=448)
        close(whole[1], ref[390:], dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_states_that_hardly_forget(tmp_path, device):
    """Scan layers whose states keep the first tokens through 300 others, in portions that start inside the convolution's
    taps: a state lost or doubled between steps moves every later row."""
    cfg = config([(scan(inner=32, state=8, conv=4, dt_rank=4), None), (scan(inner=40, state=16, conv=2, dt_rank=4), None)], width=32)
    w = weights(cfg, seed=9)
    for i in (0, 1):
        w[f"l{i}.mix.A_log"] = torch.full_like(w[f"l{i}.mix.A_log"], -8.0)
    path = write_model(tmp_path / "m", cfg, w)
    toks = tokens(320, cfg["vocab"], 14)
    ref = forward(cfg, w, toks)
    assert np.abs(ref[-20:] - forward(cfg, w, toks[60:])[-20:]).max() > 0.1 * ref.std()
    parts = cut(300, [2, 1, 3, 2, 90, 1]) + [(k, k + 1) for k in range(300, 320)]
    steps = [([("a", toks[a:b], list(range(b - a)))], []) for a, b in parts]
    for dtype in dtypes_for(device):
        got = replay(path, steps, tmp_path, device, dtype, max_tokens=320)
        # (bfloat16: a state that keeps everything also keeps every rounding of its inputs)
        close(np.concatenate([got[i] for i in range(len(steps))]), ref, dtype, 0.03)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(model, device):
    """LLM.generate (the scheduler's own portions: a 16-token step budget cuts prompts, decoded tokens share steps with
    prompt pieces, five requests over three slots) continues every prompt as the oracle's greedy loop does."""
    from nanovllm import LLM, SamplingParams
    path, cfg, w = model
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (37, 3, 18, 1, 70)]

    def greedy(p, n):
        p = list(p)
        for _ in range(n):
            p.append(int(forward(cfg, w, p)[-1].argmax()))
        return p[-n:]
    llm = LLM(path, device=device, dtype=torch.float32, max_num_seqs=3, max_num_batched_tokens=16, num_kvcache_blocks=5)
    out = llm.generate(prompts, SamplingParams(max_tokens=6, ignore_eos=True))
    assert [o["token_ids"] for o in out] == [greedy(p, 6) for p in prompts]
    assert len(llm.scheduler.block_manager.free) == 5 and len(llm.scheduler.slots.free) == 3


def test_scheduler_preempts_when_blocks_run_out(model):
    """Two requests that cannot both grow in a three-block pool: the later one is put back, runs again afterwards from
    its first token (its pages and slot hold another request's rows and state by then), and both produce what they
    produce alone."""
    from nanovllm import LLM, SamplingParams
    path, cfg, w = model
    prompts = [tokens(60, cfg["vocab"], 31), tokens(62, cfg["vocab"], 32)]
    sp = SamplingParams(max_tokens=10, ignore_eos=True)
    alone = [LLM(path, device="cpu", dtype=torch.float32, max_num_seqs=2, num_kvcache_blocks=4).generate([p], sp)[0]["token_ids"]
             for p in prompts]
    llm = LLM(path, device="cpu", dtype=torch.float32, max_num_seqs=2, num_kvcache_blocks=3)
    out = llm.generate(prompts, sp)
    assert [o["token_ids"] for o in out] == alone


def test_registry_config_and_dummy_weights(tmp_path):
    from nanovllm.models import registry
    assert registry.architecture_of({"architecture": "Tafopel"}) == "Tafopel"
    from nanovllm import LLM, SamplingParams
    bad = [[(("conv", {}), None)], [(latent(kv_from=0), None)], [(scan(), None), (latent(kv_from=0), None)],
           [(latent(), None), (latent(kv_from=0), None), (latent(kv_from=1), None)], [(scan(), dict(kind="other"))]]
    for k, layers in enumerate(bad):                # unknown kinds; readers of themselves, of a scan, of another reader
        with pytest.raises(ValueError):
            LLM(write_model(tmp_path / f"bad{k}", config(layers), {}), device="cpu", load_format="dummy")
    # a model without a checkpoint: random tensors under the checkpoint's names go through the same placement
    path = write_model(tmp_path / "dummy", config(DEFAULT), {})
    llm = LLM(path, device="cpu", dtype=torch.float32, load_format="dummy", max_num_seqs=2, num_kvcache_blocks=4)
    out = llm.generate([tokens(20, 61, 1)], SamplingParams(max_tokens=3, ignore_eos=True))
    assert len(out[0]["token_ids"]) == 3
    model = llm.model_runner.model
    # every checkpoint name is placed, none is left out, and a reader keeps no rows of its own
    names = set(model.checkpoint_tensors())
    assert names == set(weights(config(DEFAULT)))
    params = dict(model.named_parameters())
    assert all(model.load_checkpoint_tensor(params, n, t) for n, t in weights(config(DEFAULT)).items())
    assert not model.load_checkpoint_tensor(params, "l2.mix.dkv", torch.zeros(32, 48))
    rows = [m["kv_rank"] + m["rot_dim"] for (k, m), _ in DEFAULT if k == "latent_attention" and "kv_from" not in m]
    assert model.cache_bytes_per_block(64) == 64 * sum(rows) * 4


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_captured_decode_steps_equal_eager_steps(model, dtype):
    """Decode-only steps replay a hipGraph per batch-size bucket.  Three requests decode for 70 steps (a block border is
    crossed, states and convolution inputs advance inside replays, the batch shrinks from 3 to 2 to 1: three buckets,
    padding rows in the bucket of 4) with an eager prefill of a fourth request between replays; every step's logits equal
    those of an engine that runs everything eagerly."""
    from nanovllm.engine.llm_engine import LLMEngine
    from nanovllm.engine.sequence import ACTIVE, Sequence
    path, cfg, w = model
    engines = [LLMEngine(path, dtype=dtype, enforce_eager=eager, max_num_seqs=4, num_kvcache_blocks=12, max_model_len=256,
                         max_num_batched_tokens=4096) for eager in (True, False)]
    assert not engines[0].model_runner.portion_graphs and sorted(engines[1].model_runner.portion_graphs) == [1, 2, 4]
    prompts = [tokens(n, cfg["vocab"], 40 + n) for n in (50, 3, 61)]
    cont = [tokens(70, cfg["vocab"], 50 + i) for i in range(3)]
    outs = []
    for eng in engines:
        seqs, got = [], []
        for p in prompts:
            s = Sequence(p)
            s.state = ACTIVE
            assert eng.scheduler.reserve_portion(s, len(p))
            seqs.append(s)
        got.append(eng.forward_portions([(s, len(s)) for s in seqs]))
        for s in seqs:
            s.num_computed = s.num_tokens
        for step in range(70):
            live = [(i, s) for i, s in enumerate(seqs) if not (i == 1 and step >= 20) and not (i == 2 and step >= 45)]
            for i, s in live:
                s.extend([cont[i][step]])
                assert eng.scheduler.reserve_portion(s, 1)
            got.append(eng.forward_portions([(s, 1) for _, s in live]))
            for _, s in live:
                s.num_computed += 1
            if step == 30:                      # eager work between replays: another request's prompt
                extra = Sequence(tokens(40, cfg["vocab"], 99))
                extra.state = ACTIVE
                assert eng.scheduler.reserve_portion(extra, 40)
                got.append(eng.forward_portions([(extra, 40)]))
                eng.scheduler.release(extra)
        outs.append([g.float().cpu() for g in got])
    assert [a.shape for a in outs[0]] == [b.shape for b in outs[1]]
    # (float32 is the sharp comparison; in bfloat16 the split count of decode attention differs between the graph's fixed
    # table width and the eager step's, and that rounding may turn a router's near-tie)
    close(torch.cat(outs[1]).numpy(), torch.cat(outs[0]).numpy(), dtype, BF16_TIES)
