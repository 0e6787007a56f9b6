"""Larozen family — pre-normed decoder with a repeated group of layers, an
attention whose values are its keys, and an attention beside a state-space
recurrence.

N(v; w) = v / sqrt(mean(v^2) + eps) * (1 + w). The fp32 residual stream
starts as x = e = embed[token]; every layer does

    x <- x + mixer(N(x; n1));   x <- x + down(max(up N(x; n2), 0)^2)

Layers loop.start .. loop.stop-1 run loop.times times in a row with the same
weights; every pass starts with x <- W_in [x; e]. The logits are the last
norm's output times the embedding table. The layer list of config.json picks
per layer:

  * "attention"  grouped-query attention without a value projection: v = k
    as projected (biased), then q and k are rotated (neighbouring pairs of
    the leading coordinates), scores are tanh-capped; causal softmax.
  * "parallel"   two mixers read the same input, each output is RMS-normed
    with its own weight, and half their sum is the result. LEFT: causal
    attention without rotation; q and k are RMS-normed over all heads at
    once, q grows with the logarithm of the position, exp(sink_h) joins the
    softmax denominator. RIGHT: Mamba-2 — short convolution (+ bias, SiLU),
    step = softplus(dt + b), S <- exp(-exp(A) step) S + step B x^T,
    y = S^T C + D x; y silu(z) is RMS-normed in equal parts.

Serving design (what runs on the MI355X):

  * Both mixers' wide projections of a "parallel" layer are ONE GEMM
    (MaskedAttention's extra rows); the step sizes come from
    ops.narrow_linear (bf16 rows, fp32 result).
  * A tied value differs from its cached key only in the rotated
    coordinates: the value pool keeps just those, the attention kernels take
    the rest from the key row they have read for the score. The checkpoint's
    neighbouring rotary pairs become (i, i + half) pairs at load — q, k and,
    through W_o's columns, the tied values are permuted alike.
  * The recurrence is one more kind of ops.matrix_memory_scan (B in the
    place of k, C of q, x of v); memory and convolution tail are
    per-sequence state.
  * ops.residual_update_norm fuses the (plain or two-output) residual update
    with the norm that feeds the next GEMM: two launches per layer run. What
    a pass takes in is one GEMM over [x | e] rows: the update before it
    writes x's half, the embedding e's once per step, and the product is the
    new fp32 stream without a rounding in between (ops.linear_fp32).
  * Like Mugazen, the unit that owns memory is the layer RUN.

compute dtype: bf16 (serving default; positions, angles, scores, softmax,
norms, step sizes, decays, recurrent state and the residual stay fp32) or
float32 (everything fp32 — a verification mode).
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch

from .. import ops
from .llama import AttnMetadata
from .mugazen import LayerRun, layer_runs
from .volalorn import MaskedAttention, MaskedAttentionConfig, _align, _param


@dataclass
class StateSpaceConfig:
    heads: int
    vdim: int                 # value channels per head
    state: int                # state rows per head (size of B and C)
    groups: int               # B / C are shared by heads / groups heads
    conv_taps: int
    norm_groups: int          # equal parts of the gated output's norm

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def conv_channels(self) -> int:
        return self.inner + 2 * self.groups * self.state


@dataclass
class LarozenLayerConfig:
    kind: str
    attn: MaskedAttentionConfig
    space: Optional[StateSpaceConfig] = None
    ff: int = 0               # 0: no feed-forward


@dataclass
class LarozenConfig:
    name: str = "tiny-larozen"
    vocab_size: int = 512
    hidden_size: int = 128
    layers: List[LarozenLayerConfig] = field(default_factory=list)
    norm_eps: float = 1e-6
    loop_start: int = 0       # layers start .. stop-1 run `times` times
    loop_stop: int = 0
    loop_times: int = 1
    family: str = "larozen"

    @property
    def n_layers(self) -> int:
        """Cache entries: layer runs, not layers."""
        return len(self.runs())

    @property
    def max_position(self) -> int:
        return 1 << 30

    @property
    def looped(self) -> bool:
        return self.loop_stop > self.loop_start

    def runs(self) -> List[LayerRun]:
        return layer_runs(len(self.layers), self.loop_start, self.loop_stop,
                          self.loop_times)

    def _kv_shapes(self):
        mixers = [self.layers[r.layer].attn for r in self.runs()]
        return [(a.kv_heads, a.dim, a.pool_vdim) for a in mixers]

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(g * (d + dv) for g, d, dv in self._kv_shapes()
                   ) * dtype_bytes

    def state_shapes(self) -> List[Dict[str, tuple]]:
        out = []
        for r in self.runs():
            d: Dict[str, tuple] = {}
            m = self.layers[r.layer].space
            if m is not None:
                d["S"] = (m.heads, m.vdim, m.state)
                d["conv"] = (m.conv_taps - 1, m.conv_channels)
            out.append(d)
        return out

    def cache_layout(self):
        from ..engine.kvcache import HybridStateLayout
        return HybridStateLayout(self._kv_shapes(), self.state_shapes())

    def state_bytes_per_seq(self) -> int:
        return self.cache_layout().state_bytes_per_seq()


def _attention_from_dict(mx: dict, **kw) -> MaskedAttentionConfig:
    return MaskedAttentionConfig(
        heads=int(mx["heads"]), kv_heads=int(mx["kv_heads"]),
        dim=int(mx["dim"]), vdim=int(mx["vdim"]), scale=float(mx["scale"]),
        mask_kind=ops.MASK_CAUSAL, mask_size=0, qkv_bias=True, **kw)


def config_from_dict(d: dict, name: str = "larozen") -> LarozenConfig:
    """LarozenConfig from a parsed config.json."""
    layers: List[LarozenLayerConfig] = []
    for i, ld in enumerate(d["layers"]):
        kind, mx = ld["type"], ld["mixer"]
        if kind == "attention":
            rot = mx.get("rot") or {}
            dims = int(rot.get("dims", 0))
            lc = LarozenLayerConfig(kind, _attention_from_dict(
                mx, rot_dims=dims, rot_base=float(rot.get("base", 10000.0)),
                rot_pairs=True, rotate_only=True, plain_qk=dims == 0,
                tied_values=True, softcap=float(mx.get("softcap") or 0.0)))
            if lc.attn.vdim != lc.attn.dim:
                raise ValueError(f"layer {i}: values that are the keys have "
                                 "their size")
            if dims % 2 or dims > lc.attn.dim:
                raise ValueError(f"layer {i}: bad rot.dims {dims}")
        elif kind == "parallel":
            a, r = mx["left"], mx["right"]
            temp = a.get("q_temp") or {}
            every = temp.get("every", 1)
            lc = LarozenLayerConfig(kind, _attention_from_dict(
                a, row_norm=True, sink=True, out_bias=True,
                q_temp_coef=float(temp.get("coef", 0.0)),
                q_temp_every=int(every)))
            if int(every) != every or every < 1:
                raise ValueError(f"layer {i}: q_temp.every must be a positive "
                                 "whole number")
            m = lc.space = StateSpaceConfig(
                heads=int(r["heads"]), vdim=int(r["vdim"]),
                state=int(r["state"]), groups=int(r["groups"]),
                conv_taps=int(r["conv"]), norm_groups=int(r["norm_groups"]))
            if m.heads % m.groups:
                raise ValueError(f"layer {i}: heads % groups != 0")
            if m.inner % m.norm_groups:
                raise ValueError(f"layer {i}: unequal norm_groups")
            if m.conv_taps < 1:
                raise ValueError(f"layer {i}: conv must be >= 1")
        else:
            raise ValueError(f"layer {i}: unsupported mixer {kind!r}")
        if lc.attn.heads % lc.attn.kv_heads:
            raise ValueError(f"layer {i}: heads % kv_heads != 0")
        ml = ld.get("mlp")
        if ml is not None:
            if ml["kind"] != "dense":
                raise ValueError(f"layer {i}: unsupported mlp {ml['kind']!r}")
            lc.ff = int(ml["ff"])
        layers.append(lc)
    lp = d.get("loop") or {}
    cfg = LarozenConfig(
        name=name, vocab_size=int(d["vocab"]), hidden_size=int(d["width"]),
        layers=layers, norm_eps=float(d["norm"]["eps"]),
        loop_start=int(lp.get("start", 0)), loop_stop=int(lp.get("stop", 0)),
        loop_times=int(lp.get("times", 1)))
    if not 0 <= cfg.loop_start <= cfg.loop_stop <= len(layers):
        raise ValueError("loop.start .. loop.stop is not a range of layers")
    if cfg.loop_times < 1:
        raise ValueError("loop.times must be >= 1")
    return cfg


def config_from_checkpoint(path: str) -> LarozenConfig:
    with open(os.path.join(path, "config.json")) as f:
        return config_from_dict(json.load(f), name=path)


class StateSpaceMixer(torch.nn.Module):
    """Mamba-2 mixer over per-sequence state: short convolution, step-sized
    recurrence, gate before a grouped norm. Its wide projection [z | x | B |
    C] (rows of `in_rows`) is computed by the caller."""

    def __init__(self, width: int, mc: StateSpaceConfig, eps: float, dtype):
        super().__init__()
        self.mc, self.eps = mc, eps
        H, f32 = mc.heads, torch.float32
        # z | x B C, each starting 16-byte aligned (bf16)
        self.xbc_off = _align(mc.inner)
        self.in_rows = self.xbc_off + mc.conv_channels
        self.w_step = _param(H, width, dtype=dtype)
        self.step_bias = _param(H, dtype=f32)
        self.head_rate = _param(H, dtype=f32)
        self.skip = _param(H, dtype=f32)
        self.w_conv = _param(mc.conv_taps, mc.conv_channels, dtype=f32)
        self.b_conv = _param(mc.conv_channels, dtype=f32)
        self.norm_w = _param(mc.inner, dtype=f32)
        self.w_o = _param(width, mc.inner, dtype=dtype)

    @torch.no_grad()
    def load(self, get) -> torch.Tensor:
        """Returns the wide projection's rows for the caller's GEMM."""
        mc = self.mc
        w = get("in")
        rows = w.new_zeros(self.in_rows, w.size(1))
        rows[:mc.inner] = w[:mc.inner]
        rows[self.xbc_off:] = w[mc.inner:mc.inner + mc.conv_channels]
        self.w_step.copy_(w[mc.inner + mc.conv_channels:])
        self.step_bias.copy_(get("dt_bias").float())
        self.head_rate.copy_(get("A_log").float())
        self.skip.copy_(get("D").float())
        # checkpoint [channels, taps] -> tap-major [taps, channels]
        self.w_conv.copy_(get("conv").float().t())
        self.b_conv.copy_(get("conv.b").float())
        self.norm_w.copy_(get("norm").float())
        self.w_o.copy_(get("o"))
        return rows

    def forward(self, h: torch.Tensor, proj: torch.Tensor, state: dict,
                md: AttnMetadata) -> torch.Tensor:
        """h: the mixer input; proj [T, in_rows]: its wide projection."""
        mc = self.mc
        T, H, G, N = h.size(0), mc.heads, mc.groups, mc.state
        q_starts = md.query_starts if md.is_prefill else None
        q_lens = md.query_lens if md.is_prefill else None
        step = ops.narrow_linear(h, self.w_step)
        xbc = torch.empty(T, mc.conv_channels, dtype=torch.float32,
                          device=h.device)
        ops.short_conv_state(xbc, proj[:, self.xbc_off:], self.w_conv,
                             state["conv"], md.state_slots, md.seq_lens,
                             q_starts, q_lens, silu=True, bias=self.b_conv)
        b0, c0 = mc.inner, mc.inner + G * N
        y = torch.empty(T, H, mc.vdim, dtype=torch.float32, device=h.device)
        ops.matrix_memory_scan(
            ops.SCAN_SSD, y, xbc[:, c0:].view(T, G, N),
            xbc[:, b0:c0].view(T, G, N), xbc[:, :b0].view(T, H, mc.vdim),
            step, self.step_bias, self.head_rate, None, 1.0, 0.0, state["S"],
            None, None, md.state_slots, md.seq_lens, q_starts, q_lens,
            skip=self.skip)
        out = torch.empty(T, mc.inner, dtype=h.dtype, device=h.device)
        ops.gate_group_rmsnorm(out, y.view(T, mc.inner), self.norm_w,
                               proj[:, :mc.inner], mc.norm_groups, self.eps)
        return ops.linear(out, self.w_o)


class SquaredReluFeedForward(torch.nn.Module):
    """down( max(up h, 0)^2 )."""

    def __init__(self, width: int, ff: int, dtype):
        super().__init__()
        self.up = _param(ff, width, dtype=dtype)
        self.down = _param(width, ff, dtype=dtype)

    @torch.no_grad()
    def load(self, get):
        self.up.copy_(get("up"))
        self.down.copy_(get("down"))

    def forward(self, h):
        z = ops.linear(h, self.up)
        act = torch.empty_like(z)
        ops.relu_square(act, z)
        return ops.linear(act, self.down)


class LarozenLayer(torch.nn.Module):
    def __init__(self, cfg: LarozenConfig, lc: LarozenLayerConfig, dtype):
        super().__init__()
        W, f32 = cfg.hidden_size, torch.float32
        self.lc = lc
        # norm weights are kept as 1 + w
        self.norm1 = _param(W, dtype=f32)
        if lc.space is None:
            self.mix = MaskedAttention(W, lc.attn, cfg.norm_eps, dtype)
            self.space = None
        else:
            self.space = StateSpaceMixer(W, lc.space, cfg.norm_eps, dtype)
            self.mix = MaskedAttention(W, lc.attn, cfg.norm_eps, dtype,
                                       extra_rows=self.space.in_rows)
            # the two outputs' norm weights, halved: the sum is half and half
            self.out_left = _param(W, dtype=f32)
            self.out_right = _param(W, dtype=f32)
        self.norm2, self.mlp = None, None
        if lc.ff > 0:
            self.norm2 = _param(W, dtype=f32)
            self.mlp = SquaredReluFeedForward(W, lc.ff, dtype)


class LarozenForCausalLM(torch.nn.Module):
    def __init__(self, cfg: LarozenConfig, device="cpu", tp_rank: int = 0,
                 tp_size: int = 1, seed: int = 0, dtype=torch.bfloat16):
        super().__init__()
        if tp_size != 1:
            raise ValueError("Larozen: tensor parallelism is not implemented")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Larozen: unsupported compute dtype {dtype}")
        self.cfg = cfg
        self.dtype = dtype
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.runs = cfg.runs()
        W = cfg.hidden_size
        with torch.device(device):
            self.embed = _param(cfg.vocab_size, W, dtype=dtype)
            self.loop_in = (_param(W, 2 * W, dtype=dtype) if cfg.looped
                            else None)
            self.layers = torch.nn.ModuleList(
                [LarozenLayer(cfg, lc, dtype) for lc in cfg.layers])
            self.final_norm = _param(W, dtype=torch.float32)
        self.random_init(seed)
        # test hook: when a list, receives the residual after every layer run
        self.residual_trace: Optional[list] = None

    @torch.no_grad()
    def random_init(self, seed: int = 0):
        gen = torch.Generator(device=self.embed.device).manual_seed(seed)

        def normal(p, std, mean=0.0):
            p.copy_((mean + torch.randn(p.shape, generator=gen,
                                        device=p.device, dtype=torch.float32)
                     * std).to(p.dtype))

        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("out_left", "out_right"):
                p.fill_(0.5)
            elif leaf in ("b_in", "b_o", "b_conv"):
                normal(p, 0.1)
            elif leaf == "sink":
                normal(p, 0.5)
            elif leaf == "head_rate":
                normal(p, 0.5, -0.5)
            elif leaf == "step_bias":
                normal(p, 0.5, -2.0)
            elif leaf == "w_conv":
                normal(p, 0.5)
            elif p.dim() >= 2:
                normal(p, 1.0 / p.size(-1) ** 0.5)
            else:
                p.fill_(1.0)                      # norm weights, skips
        normal(self.embed, 1.0)

    def pack_decode_weights(self):
        """Projections run on hipBLASLt in both phases; nothing to repack."""

    @torch.no_grad()
    def load_safetensors(self, path: str):
        from safetensors.torch import load_file
        import glob

        files = sorted(glob.glob(os.path.join(path, "*.safetensors")))
        if not files:
            raise FileNotFoundError(f"no safetensors under {path}")
        sd: Dict[str, torch.Tensor] = {}
        for f in files:
            sd.update(load_file(f))
        self.load_state(sd)

    @torch.no_grad()
    def load_state(self, sd: Dict[str, torch.Tensor]):
        """Copy checkpoint tensors (embed, loop.in, l<i>.norm1/2, l<i>.mix.*,
        l<i>.mlp.*, final.norm) into the fused serving layout."""
        dev, dt = self.embed.device, self.dtype

        def getter(prefix):
            def get(name):
                return sd[prefix + name].to(device=dev, dtype=dt)
            return get

        top = getter("")
        self.embed.copy_(top("embed"))
        if self.loop_in is not None:
            self.loop_in.copy_(top("loop.in"))
        self.final_norm.copy_(1.0 + top("final.norm").float())
        for i, layer in enumerate(self.layers):
            g = getter(f"l{i}.")
            layer.norm1.copy_(1.0 + g("norm1").float())
            if layer.space is None:
                layer.mix.load(getter(f"l{i}.mix."))
            else:
                rows = layer.space.load(getter(f"l{i}.mix.right."))
                layer.mix.load(getter(f"l{i}.mix.left."), extra=rows)
                layer.out_left.copy_(0.5 * g("mix.left.out").float())
                layer.out_right.copy_(0.5 * g("mix.right.out").float())
            if layer.mlp is not None:
                layer.norm2.copy_(1.0 + g("norm2").float())
                layer.mlp.load(getter(f"l{i}.mlp."))

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor, md: AttnMetadata,
                kv_caches: List, last_rows: Optional[torch.Tensor] = None
                ) -> torch.Tensor:
        cfg, eps, W = self.cfg, self.cfg.norm_eps, self.cfg.hidden_size
        if md.state_slots is None:
            raise ValueError("Larozen needs per-sequence state slots")
        T, dev = input_ids.size(0), input_ids.device
        x = torch.empty(T, W, dtype=torch.float32, device=dev)
        # rows [x | e], the input of a pass's first projection
        xe = (torch.empty(T, 2 * W, dtype=self.dtype, device=dev)
              if cfg.looped else None)
        ops.embed_rows(input_ids, self.embed, x,
                       None if xe is None else xe[:, W:])

        def update(x, kind, y=None, w=None, y2=None, w2=None, norm=None,
                   cast=None):
            """One residual update of x, then N(x; norm) for the next GEMM
            (returned), or x itself into `cast`, or nothing."""
            out = cast
            if norm is not None:
                out = torch.empty(x.size(0), W, dtype=self.dtype, device=dev)
            ops.residual_update_norm(x, y, kind, None, None, w, eps, norm,
                                     None, out, rms_norm=True, y2=y2,
                                     rms_w2=w2)
            return out

        n = len(self.runs)
        first = self.runs[0]
        h = None
        if first.enters:
            ops.embed_rows(input_ids, self.embed, None, xe[:, :W])
        else:
            h = update(x, ops.UPDATE_NONE,
                       norm=self.layers[first.layer].norm1)
        tables: dict = {}      # rotary setting -> this step's cos/sin rows
        for r, run in enumerate(self.runs):
            layer = self.layers[run.layer]
            k_cache, v_cache, state = kv_caches[r]
            if run.enters:
                x = ops.linear_fp32(xe, self.loop_in)
                h = update(x, ops.UPDATE_NONE, norm=layer.norm1)
            nxt = self.runs[r + 1] if r + 1 < n else None
            # what the layer's last update hands on
            tail: dict = {}
            if nxt is None:
                # only the wanted rows need the final norm
                if last_rows is None:
                    tail["norm"] = self.final_norm
            elif nxt.enters:
                tail["cast"] = xe[:, :W]
            else:
                tail["norm"] = self.layers[nxt.layer].norm1
            after_mix = tail if layer.mlp is None else {"norm": layer.norm2}
            if layer.space is None:
                y = layer.mix(h, k_cache, v_cache, md, tables)
                h = update(x, ops.UPDATE_ADD, y, **after_mix)
            else:
                y, wide = layer.mix(h, k_cache, v_cache, md)
                y2 = layer.space(h, wide, state, md)
                h = update(x, ops.UPDATE_UNIT_RMS, y, layer.out_left, y2,
                           layer.out_right, **after_mix)
            if layer.mlp is not None:
                h = update(x, ops.UPDATE_ADD, layer.mlp(h), **tail)
            if self.residual_trace is not None:
                self.residual_trace.append(x.clone())
        if last_rows is not None:
            h = update(x[last_rows], ops.UPDATE_NONE, norm=self.final_norm)
        return ops.linear(h, self.embed).float()


def _tiny(name: str) -> LarozenConfig:
    tied = MaskedAttentionConfig(
        heads=4, kv_heads=2, dim=32, vdim=32, scale=32 ** -0.5,
        mask_kind=ops.MASK_CAUSAL, mask_size=0, qkv_bias=True, rot_dims=16,
        rot_base=50000.0, rot_pairs=True, rotate_only=True, tied_values=True,
        softcap=20.0)
    left = MaskedAttentionConfig(
        heads=4, kv_heads=1, dim=32, vdim=32, scale=32 ** -0.5,
        mask_kind=ops.MASK_CAUSAL, mask_size=0, qkv_bias=True, row_norm=True,
        sink=True, out_bias=True, q_temp_coef=0.3, q_temp_every=64)
    right = StateSpaceConfig(heads=4, vdim=32, state=32, groups=2,
                             conv_taps=4, norm_groups=4)
    layers = [LarozenLayerConfig("attention", tied, ff=256),
              LarozenLayerConfig("parallel", left, right, ff=256),
              LarozenLayerConfig("attention", tied, ff=256)]
    return LarozenConfig(name=name, vocab_size=512, hidden_size=128,
                         layers=layers, norm_eps=1e-5, loop_start=1,
                         loop_stop=3, loop_times=2)


LAROZEN_CONFIGS: Dict[str, LarozenConfig] = {
    "tiny-larozen": _tiny("tiny-larozen"),
}


def make_larozen_instance(name: str, device: str, engine_cfg,
                          weights_path: Optional[str] = None):
    """ModelInstance over a Larozen model (engine factory hook): a named
    random-init config, or a checkpoint directory."""
    from ..engine.llm import ModelInstance

    cfg = (config_from_checkpoint(weights_path) if weights_path
           else LAROZEN_CONFIGS[name])
    if device.startswith("cuda") and not (
            ops.gated_available() and ops.masked_available()
            and ops.recurrent_available()):
        raise RuntimeError(
            "GPU engine requires the gfx950 gated, masked-attention and "
            "recurrent extensions (python -m agentainer_amd.ops.build gated "
            "masked recurrent)")
    return ModelInstance(name, cfg, device, engine_cfg,
                         weights_path=weights_path,
                         model_cls=LarozenForCausalLM)
