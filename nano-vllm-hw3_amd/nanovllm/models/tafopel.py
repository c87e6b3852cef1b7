"""Tafopel: a decoder-only model whose layers are listed one by one in config.json.  A layer has one norm whose output both
its mixer and its feed-forward read (a parallel block on a float32 residual, layer norms with a weight and no bias).  The
mixer is latent attention - queries through a latent of their own, one rotated key part shared by the heads on a frequency
table stretched for long contexts, a learned sink per head; a layer may read another layer's cached rows - or a selective
scan ("mamba1").  The feed-forward is dense with a tanh-GELU gate, or a mixture of squared-ReLU experts behind a sigmoid
router whose weights multiply what the experts read, with a shared expert scaled by a gate of its own; it may be absent.

Read from config.json: vocab, width, norm.eps, and per layer
  {type, mixer: {heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, rot: {dims, base, scaling: {factor, original, fast, slow}}, kv_from} |
                {inner, state, conv, dt_rank},
   mlp: null | {kind: dense, ff} | {kind: moe, expert: {ff}, router: {experts, top}, shared: null | {ff}}}.
Checkpoint tensors: embed, final.norm, head, and per layer l<i>.{norm1, mix.*, mlp.*}.

The model is stepped with portions of sequences (nanovllm.seq_ops.StepContext).  It owns, per latent layer with a
down-projection, one paged cache of [latent | rotated key part] rows (all layers share a sequence's block table) and, per
state slot, every scan layer's float32 state and its convolution's last inputs."""
import re

import torch
from torch import nn

from nanovllm import hy_ops
from nanovllm.layers.f32_product import F32Product
from nanovllm.layers.feedforward import GatedMLP, ReluSquaredMLP, RoutedExperts
from nanovllm.layers.latent_attention import LatentAttention
from nanovllm.layers.parallel_block import ParallelBlock
from nanovllm.layers.selective_scan import SelectiveScan


def make_mixer(cfg, spec, earlier):
    W, m = cfg.hidden_size, spec["mixer"]
    if spec["type"] == "mamba1":
        return SelectiveScan(W, m["inner"], m["state"], m["conv"], m["dt_rank"])
    if spec["type"] != "latent_attention":
        raise ValueError(f"unknown mixer type {spec['type']!r}")
    src, source = m.get("kv_from"), None
    if src is not None:
        if not (0 <= src < len(earlier) and isinstance(earlier[src].block.mixer, LatentAttention)):
            raise ValueError(f"kv_from: {src} is not an earlier latent layer")
        source = earlier[src].block.mixer
        if source.kv_source is not None:
            raise ValueError(f"kv_from: layer {src} reads another layer's rows itself")
    # a reader's row layout and rotation are its source's (config.json may repeat them)
    rot = m.get("rot") or ({} if source is None else dict(dims=source.rot_dims, base=source.rot_base, scaling=source.rot_scaling))
    rot_dim = m.get("rot_dim", 0 if source is None else source.rot_dim)
    return LatentAttention(W, m["heads"], m["dim"], m["vdim"], m["kv_rank"] if source is None else m.get("kv_rank", source.kv_rank),
                           m["scale"], cfg.norm_eps, rot_dim=rot_dim, rot_dims=rot.get("dims", rot_dim),
                           rot_base=rot.get("base", 10000.0), q_rank=m["q_rank"], rot_scaling=rot.get("scaling"), sink=True,
                           kv_source=source)


def make_mlp(cfg, mlp):
    W = cfg.hidden_size
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return GatedMLP(W, mlp["ff"], "gelu_tanh_glu")
    if mlp["kind"] != "moe":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    r, sh = mlp["router"], mlp.get("shared")
    return RoutedExperts(W, r["experts"], r["top"], mlp["expert"]["ff"], shared=ReluSquaredMLP(W, sh["ff"]) if sh else None,
                         score="sigmoid", renorm=False, act="relu_sq", weight_in=True, shared_gate=bool(sh))


class TafopelLayer(nn.Module):
    def __init__(self, cfg, spec, earlier):
        super().__init__()
        self.norm = nn.Parameter(torch.ones(cfg.hidden_size), requires_grad=False)
        self.block = ParallelBlock(make_mixer(cfg, spec, earlier), make_mlp(cfg, spec.get("mlp")))


class TafopelForCausalLM(nn.Module):
    runs_portions = True           # stepped with portions; owns its caches and per-sequence state
    default_block_size = 64
    native_library = ("hymix", "seqmix")      # norms and the scan; convolution, latent attention and experts

    @staticmethod
    def normalize_config(d: dict) -> dict:
        d = dict(d)
        d["vocab_size"], d["hidden_size"] = d["vocab"], d["width"]
        d["max_position_embeddings"] = d.get("max_positions", 1 << 20)
        d["norm_eps"] = d["norm"]["eps"]
        d.setdefault("torch_dtype", "bfloat16")
        return d

    def __init__(self, cfg):
        super().__init__()
        self.cfg = cfg
        W = cfg.hidden_size
        self.dtype = torch.get_default_dtype()
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, W), requires_grad=False)
        layers = []
        for spec in cfg.layers:
            layers.append(TafopelLayer(cfg, spec, layers))
        self.layers = nn.ModuleList(layers)
        self.final_norm = nn.Parameter(torch.ones(W), requires_grad=False)
        self.head = nn.Parameter(torch.empty(cfg.vocab_size, W), requires_grad=False)
        self.logits_product = F32Product()

    # ------------------------------------------------------------------ checkpoint names
    _SIMPLE = {"norm1": "norm", "mix.o": "block.mixer.o_proj",
               "mix.dq.norm": "block.mixer.q_latent_norm", "mix.uq": "block.mixer.uq", "mix.dkv.norm": "block.mixer.latent_norm",
               "mix.sink": "block.mixer.sink",
               "mix.in": "block.mixer.in_proj", "mix.conv": "block.mixer.conv.weight", "mix.conv.b": "block.mixer.conv.bias",
               "mix.x": "block.mixer.x_proj", "mix.dt": "block.mixer.dt_proj", "mix.dt.b": "block.mixer.dt_bias", "mix.D": "block.mixer.D",
               "mlp.down": "block.mlp.down", "mlp.router": "block.mlp.router", "mlp.shared.up": "block.mlp.shared.up",
               "mlp.shared.down": "block.mlp.shared.down", "mlp.shared.sg": "block.mlp.shared_gate"}

    def load_checkpoint_tensor(self, params, name, tensor):
        """Place one checkpoint tensor; returns False for a name this model does not know."""
        top = {"embed": "embed", "final.norm": "final_norm", "head": "head"}
        if name in top:
            params[top[name]].data.copy_(tensor)
            return True
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        if not m or int(m.group(1)) >= len(self.layers):
            return False
        i, rest = int(m.group(1)), m.group(2)
        mx, mlp = self.layers[i].block.mixer, self.layers[i].block.mlp
        if rest in self._SIMPLE:
            p = params.get(f"layers.{i}.{self._SIMPLE[rest]}")
            if p is None:
                return False
            p.data.copy_(tensor.reshape(p.shape))
            return True
        if isinstance(mx, SelectiveScan) and rest == "mix.A_log":
            mx.A.data.copy_(-torch.exp(tensor.to(mx.A.device).float()))
        elif isinstance(mx, LatentAttention) and rest == "mix.dq":
            mx.qc_proj.data[:mx.q_rows].copy_(tensor)
        elif isinstance(mx, LatentAttention) and rest == "mix.dkv" and mx.kv_source is None:
            mx.qc_proj.data[mx.q_rows:].copy_(tensor)
        elif isinstance(mx, LatentAttention) and rest == "mix.uk":
            mx.uk.data.copy_(tensor.view(mx.heads, mx.dim, mx.kv_rank))
        elif isinstance(mx, LatentAttention) and rest == "mix.uv":
            mx.uv.data.copy_(tensor.view(mx.heads, mx.vdim, mx.kv_rank).transpose(1, 2))
        elif isinstance(mlp, GatedMLP) and rest in ("mlp.gate", "mlp.up"):
            mlp.gate_up.data[(mlp.ff if rest == "mlp.up" else 0):][:mlp.ff].copy_(tensor)
        else:
            e = re.fullmatch(r"mlp\.e(\d+)\.(up|down)", rest)
            if not e or not isinstance(mlp, RoutedExperts) or int(e.group(1)) >= mlp.experts:
                return False
            w = mlp.w_gu if e.group(2) == "up" else mlp.w_down
            w.data[int(e.group(1))].copy_(tensor)
        return True

    def checkpoint_tensors(self, seed=0, std=0.05):
        """Random tensors with the checkpoint's names and shapes (benchmarks and tests without a checkpoint), drawn in
        a fixed order from one seeded generator on the model's device."""
        cfg, dev = self.cfg, self.embed.device
        g = torch.Generator(device=dev).manual_seed(seed)
        W = cfg.hidden_size

        def rnd(*shape, s=std):
            return torch.randn(*shape, generator=g, device=dev, dtype=torch.float32) * s
        t = {"embed": rnd(cfg.vocab_size, W, s=1.0), "final.norm": 1 + rnd(W), "head": rnd(cfg.vocab_size, W, s=W ** -0.5)}
        for i, (spec, layer) in enumerate(zip(cfg.layers, self.layers)):
            p, mx = f"l{i}.", layer.block.mixer
            t[p + "norm1"] = 1 + rnd(W)
            if isinstance(mx, SelectiveScan):
                C, N, R = mx.inner, mx.states, mx.dt_rank
                t.update({p + "mix.in": rnd(2 * C, W, s=W ** -0.5), p + "mix.conv": rnd(C, mx.taps, s=mx.taps ** -0.5),
                          p + "mix.conv.b": rnd(C, s=0.1), p + "mix.x": rnd(R + 2 * N, C, s=C ** -0.5),
                          p + "mix.dt": rnd(C, R, s=R ** -0.5), p + "mix.dt.b": rnd(C) - 3.0,
                          p + "mix.A_log": torch.log(torch.arange(1, N + 1, device=dev).float()).expand(C, N) + rnd(C, N),
                          p + "mix.D": 1 + rnd(C), p + "mix.o": rnd(W, C, s=C ** -0.5)})
            else:
                H, D, V, R, Rd, Q = mx.heads, mx.dim, mx.vdim, mx.kv_rank, mx.rot_dim, mx.q_rank
                t.update({p + "mix.dq": rnd(Q, W, s=W ** -0.5), p + "mix.dq.norm": 1 + rnd(Q, s=0.2),
                          p + "mix.uq": rnd(H * (D + Rd), Q, s=Q ** -0.5), p + "mix.uk": rnd(H * D, R, s=R ** -0.5),
                          p + "mix.uv": rnd(H * V, R, s=R ** -0.5), p + "mix.sink": rnd(H, s=1.0),
                          p + "mix.o": rnd(W, H * V, s=(H * V) ** -0.5)})
                if mx.kv_source is None:
                    t.update({p + "mix.dkv": rnd(R + Rd, W, s=W ** -0.5), p + "mix.dkv.norm": 1 + rnd(R, s=0.2)})
            mlp = spec.get("mlp")
            if mlp is None:
                continue
            if mlp["kind"] == "dense":
                ff = mlp["ff"]
                t.update({p + "mlp.gate": rnd(ff, W, s=W ** -0.5), p + "mlp.up": rnd(ff, W, s=W ** -0.5),
                          p + "mlp.down": rnd(W, ff, s=ff ** -0.5)})
                continue
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            t[p + "mlp.router"] = rnd(E, W, s=2 * W ** -0.5)
            for e in range(E):
                t.update({f"{p}mlp.e{e}.up": rnd(ff, W, s=W ** -0.5), f"{p}mlp.e{e}.down": rnd(W, ff, s=ff ** -0.5)})
            if mlp.get("shared"):
                fs = mlp["shared"]["ff"]
                t.update({p + "mlp.shared.up": rnd(fs, W, s=W ** -0.5), p + "mlp.shared.down": rnd(W, fs, s=fs ** -0.5),
                          p + "mlp.shared.sg": rnd(1, W, s=W ** -0.5)})
        return {k: v.to(torch.bfloat16) for k, v in t.items()}

    # ------------------------------------------------------------------ cache and state
    def _mixers(self, kind):
        return [l.block.mixer for l in self.layers if isinstance(l.block.mixer, kind)]

    def cache_bytes_per_block(self, block_size):
        return sum(block_size * mx.cache_bytes_per_token(self.dtype.itemsize) for mx in self._mixers(LatentAttention))

    def state_bytes_per_slot(self):
        return sum(mx.state_bytes_per_slot(self.dtype.itemsize) for mx in self._mixers(SelectiveScan))

    def allocate_cache(self, num_blocks, block_size, num_slots, device):
        """One cache of [latent | rotated key part] rows per latent layer with a down-projection (a reader takes its source's;
        all share the sequences' block tables); per state slot one float32 state and the convolution's last inputs per scan layer."""
        self.num_slots = num_slots
        for mx in self._mixers(LatentAttention):       # in order: a reader's source comes before it
            mx.allocate(0, num_blocks, block_size, self.dtype, device)
        for mx in self._mixers(SelectiveScan):
            mx.allocate(num_slots, self.dtype, device)

    def workspaces(self):
        """Scratch buffers that captured decode graphs address."""
        from nanovllm import _seqmix
        return [_seqmix.decode_workspace]

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, trace=None):
        """input_ids int64 [T], positions int32 [T] (the step's context is seq_ops.get_step()) -> final-normed hidden
        [T, width].  ``trace``: a list that receives the residual after every layer (debugging)."""
        dt, eps, n = self.dtype, self.cfg.norm_eps, len(self.layers)
        x, h = hy_ops.layer_norm_residual(None, self.embed, self.layers[0].norm, eps, dt, ids=input_ids)
        for i, layer in enumerate(self.layers):
            y, routed = layer.block(h)
            # the write of this block and the norm in front of the next one (behind the last: the final norm), in one launch
            x, h = hy_ops.layer_norm_residual(x, y, self.layers[i + 1].norm if i + 1 < n else self.final_norm, eps, dt, routed=routed)
            if trace is not None:
                trace.append(x.clone())
        return h

    def compute_logits(self, hidden_states):
        """float32 logits of the given rows: products of the stored values, float32 accumulation AND output."""
        return self.logits_product(hidden_states, self.head)
