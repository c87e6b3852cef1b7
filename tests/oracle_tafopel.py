"""Plain restatement of the Tafopel design in float64 torch: one function per mechanism, whole sequences, no cache, no
batching.  It shares no code with the package; the tests compare the engine and its kernels against it.

A model is (cfg, tensors): cfg the parsed config.json, tensors a dict name -> tensor under the checkpoint's names."""
import math

import torch

F64 = torch.float64


def layer_norm(x, w, eps):
    """Mean removed, divided by the root of the mean squared deviation plus eps, times w; no bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return torch.clamp(z, min=0) ** 2


# ------------------------------------------------------------------------------------------ latent attention
def rotary_table(rot):
    """rot = {dims, base, scaling?} -> (frequencies [dims/2], factor on cos and sin).  ``scaling`` divides the frequencies
    of slowly turning pairs by its factor, keeps those of fast pairs, and runs a linear ramp over the pair index between."""
    dims, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64), 1.0

    def where(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(where(sc["fast"])), 0), min(math.ceil(where(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_interleaved(x, freqs, mag):
    """x [T, ..., D], row t at position t: channels (2i, 2i+1), i < len(freqs), turned by t * freqs[i]."""
    T, n = x.shape[0], freqs.numel()
    ang = (torch.arange(T, dtype=F64)[:, None] * freqs[None, :]).reshape([T] + [1] * (x.dim() - 2) + [n])
    c, s = torch.cos(ang) * mag, torch.sin(ang) * mag
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    out = x.clone()
    out[..., 0:2 * n:2], out[..., 1:2 * n:2] = u * c - v * s, v * c + u * s
    return out


def latent_rows(h, p, m, eps):
    """What a latent layer caches: the normed latent c [T, kv_rank] and the rotated key part [T, rot_dim]."""
    freqs, mag = rotary_table(m["rot"])
    d = h @ p["mix.dkv"].T
    return rms_norm(d[:, :m["kv_rank"]], p["mix.dkv.norm"], eps), rotate_interleaved(d[:, m["kv_rank"]:], freqs, mag)


def sink_softmax(s, sink):
    """s [..., keys] and one more score whose weight is counted in the denominator only."""
    mx = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - mx)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - mx))


def latent_attention(h, c, kr, p, m, eps):
    """Queries through a normed latent of their own; keys and values up-projected from c, one rotated key part for all
    heads; causal softmax with a sink per head."""
    T = h.shape[0]
    H, D, Rd, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    freqs, mag = rotary_table(m["rot"])
    q = (rms_norm(h @ p["mix.dq"].T, p["mix.dq.norm"], eps) @ p["mix.uq"].T).reshape(T, H, D + Rd)
    qr = rotate_interleaved(q[..., D:], freqs, mag)
    k = (c @ p["mix.uk"].T).reshape(T, H, D)
    v = (c @ p["mix.uv"].T).reshape(T, H, V)
    i = torch.arange(T)
    o = torch.zeros(T, H, V, dtype=F64)
    for hh in range(H):
        s = (q[:, hh, :D] @ k[:, hh].T + qr[:, hh] @ kr.T) * m["scale"]
        s = s.masked_fill(i[:, None] < i[None, :], float("-inf"))
        o[:, hh] = sink_softmax(s, p["mix.sink"][hh]) @ v[:, hh]
    return o.reshape(T, H * V) @ p["mix.o"].T


# ------------------------------------------------------------------------------------------ selective scan
def causal_conv(x, w, b):
    """Per channel: sum over the last taps inputs (zeros before the start; the last column meets the current one) + b."""
    T, taps = x.shape[0], w.shape[1]
    out = b.expand_as(x).clone()
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            out[back:] += w[:, j] * x[:T - back]
    return out


def selective_scan(x, dt, A, B, C, D, S0=None):
    """S_t[c, n] = exp(dt_c A[c, n]) S_(t-1)[c, n] + dt_c x_c B_n, y_c = sum_n S_t[c, n] C_n + D_c x_c.
    x, dt [T, channels], A [channels, N], B, C [T, N] -> (y [T, channels], S)."""
    S = torch.zeros(A.shape, dtype=F64) if S0 is None else S0.clone()
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba_mixer(h, p, m):
    inner, R, N = m["inner"], m["dt_rank"], m["state"]
    xz = h @ p["mix.in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, p["mix.conv"], p["mix.conv.b"]))
    d = x @ p["mix.x"].T
    dt = softplus(d[:, :R] @ p["mix.dt"].T + p["mix.dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(p["mix.A_log"]), d[:, R:R + N], d[:, R + N:], p["mix.D"])
    return (y * silu(z)) @ p["mix.o"].T


# ------------------------------------------------------------------------------------------ feed-forward
def dense(h, p):
    return (gelu_tanh(h @ p["mlp.gate"].T) * (h @ p["mlp.up"].T)) @ p["mlp.down"].T


def expert(h, p, name):
    return relu_squared(h @ p[name + ".up"].T) @ p[name + ".down"].T


def route(h, w, top):
    """Sigmoid scores; the ``top`` largest are chosen and weigh as they are."""
    val, idx = torch.sigmoid(h @ w.T).topk(top, -1)
    return idx, val


def mixture(h, p, mlp):
    """The weight multiplies what an expert reads; a shared expert is added, scaled by one sigmoid gate per token."""
    idx, wts = route(h, p["mlp.router"], mlp["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(idx[t].tolist(), wts[t]):
            y[t] += expert(w * h[t], p, f"mlp.e{e}")
    if mlp.get("shared"):
        y = y + torch.sigmoid(h @ p["mlp.shared.sg"].T) * expert(h, p, "mlp.shared")
    return y


# ------------------------------------------------------------------------------------------ model
def forward(cfg, tensors, tokens):
    """tokens [T] of one sequence -> (float64 logits [T, vocab], the residual after every layer [L, T, W])."""
    t = {k: v.to(F64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    trace, kept = [], {}
    for i, spec in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", spec["mixer"]
        p = {k[len(pre):]: v for k, v in t.items() if k.startswith(pre)}
        h = layer_norm(x, p["norm1"], eps)
        if spec["type"] == "mamba1":
            y = mamba_mixer(h, p, m)
        else:
            src = m.get("kv_from")
            if src is None:
                kept[i] = latent_rows(h, p, m, eps)
            y = latent_attention(h, *kept[i if src is None else src], p, m, eps)
        mlp = spec.get("mlp")
        if mlp is not None:
            y = y + (dense(h, p) if mlp["kind"] == "dense" else mixture(h, p, mlp))
        x = x + y
        trace.append(x.clone())
    return layer_norm(x, t["final.norm"], eps) @ t["head"].T, torch.stack(trace)
