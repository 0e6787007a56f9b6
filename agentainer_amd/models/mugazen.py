"""Mugazen family — sandwich-normed decoder with a repeated group of layers,
a gated delta-rule mixer and a latent-attention mixer with softmax sinks.

N(v; w) is the RMS norm v / sqrt(mean(v^2) + eps) * w. The fp32 residual
stream x starts as N(scale * embed[token] + pos[position]), and every layer
norms its sublayers on both sides:

    x <- x + N(mixer(N(x; n1)); n1b);   x <- x + N(ff(N(x; n2)); n2b)

Layers loop.start .. loop.stop-1 run loop.times times in a row with the
same weights; pass t starts with x <- x + [t > 0] e + step[t], e being the
stream as it was before the first layer. The layer list of config.json
picks per layer:

  * "delta"            gated delta rule: q, k, v pass a short causal
    convolution + SiLU, q and k become unit vectors; one decay
    g = exp(-exp(A) softplus(W_a h + b)) and one write strength
    beta = sigmoid(W_b h) per head; S <- g S; u = beta (v - S^T k);
    S <- S + k u^T; o = S^T q; per-head RMS norm, SiLU output gate.
  * "latent_attention" position-free causal attention: queries through an
    RMS-normed latent, keys and values expanded from one cached RMS-normed
    latent per token; exp(sink_h) joins head h's softmax denominator; one
    sigmoid gate per head.

and a feed-forward: a dense clamped gated unit, or routed SiLU-gated
experts weighed by the softmax over the chosen experts' logits.

Serving design (what runs on the MI355X):

  * The unit that owns memory is the layer RUN, not the layer: a looped
    layer has one latent pool / recurrent state per pass, laid out as
    consecutive entries of one HybridStateLayout, so page tables, slots,
    offload and restore work as for any other family.
  * ops.residual_update_norm fuses the norm after a sublayer, the fp32
    residual update, what a pass takes in before its first layer, and the
    norm that feeds the next GEMM: two launches per layer run.
  * Latent attention is lelitar.LatentAttention (latent basis, K = V = the
    cached rows); sink and head gate are applied where the kernels
    normalize the weighted sum.
  * The delta rule is pekarax.MatrixMemoryMixer; its per-head decay is
    evaluated inside the scan kernel from fp32 pre-activations.
  * Routers, decays and write strengths come from ops.narrow_linear (bf16
    rows, fp32 result).

compute dtype: bf16 (serving default; positions, scores, softmax, norms,
routers, recurrent state and the residual stay fp32) or float32 (everything
fp32 — a verification mode).
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Dict, List, NamedTuple, Optional

import torch

from .. import ops
from .lelitar import (CAUSAL_WINDOW, GatedFeedForward, LatentAttention,
                      LatentMixerConfig)
from .llama import AttnMetadata
from .pekarax import MatrixMemoryConfig, MatrixMemoryMixer
from .sipelorn import GroupedSigmoidExperts, SipelornFeedForwardConfig
from .volalorn import _param

UNIT_SLOPE = 1.702       # sigmoid slope of the dense clamped unit


@dataclass
class MugazenFeedForwardConfig:
    kind: str                 # "dense" | "moe"
    ff: int                   # inner size (per expert for moe)
    limit: float = 0.0        # dense: gate <= limit, |up| <= limit
    experts: int = 0
    top: int = 0


@dataclass
class MugazenLayerConfig:
    kind: str
    delta: Optional[MatrixMemoryConfig] = None
    latent: Optional[LatentMixerConfig] = None
    mlp: Optional[MugazenFeedForwardConfig] = None


class LayerRun(NamedTuple):
    """One execution of a layer; its index in the run list is the index of
    its cache entry."""
    layer: int
    loop_pass: Optional[int]  # None outside the repeated group
    enters: bool              # first layer of its pass


def layer_runs(n: int, start: int, stop: int, times: int) -> List[LayerRun]:
    """Order in which n layers run when start .. stop-1 run `times` times in
    a row (start == stop: no repeated group)."""
    if stop <= start:
        return [LayerRun(i, None, False) for i in range(n)]
    return ([LayerRun(i, None, False) for i in range(start)]
            + [LayerRun(i, t, i == start) for t in range(times)
               for i in range(start, stop)]
            + [LayerRun(i, None, False) for i in range(stop, n)])


@dataclass
class MugazenConfig:
    name: str = "tiny-mugazen"
    vocab_size: int = 512
    hidden_size: int = 128
    layers: List[MugazenLayerConfig] = field(default_factory=list)
    norm_eps: float = 1e-6
    embed_scale: float = 1.0
    max_positions: int = 2048
    loop_start: int = 0       # layers start .. stop-1 run `times` times
    loop_stop: int = 0
    loop_times: int = 1
    family: str = "mugazen"

    @property
    def n_layers(self) -> int:
        """Cache entries: layer runs, not layers."""
        return len(self.runs())

    @property
    def max_position(self) -> int:
        return self.max_positions  # rows of the learned position table

    @property
    def looped(self) -> bool:
        return self.loop_stop > self.loop_start

    def runs(self) -> List[LayerRun]:
        return layer_runs(len(self.layers), self.loop_start, self.loop_stop,
                          self.loop_times)

    def _kv_shapes(self):
        ls = [self.layers[r.layer] for r in self.runs()]
        return [None if l.latent is None else (l.latent.padded_rank,)
                for l in ls]

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(s[0] for s in self._kv_shapes() if s) * dtype_bytes

    def state_shapes(self) -> List[Dict[str, tuple]]:
        out = []
        for r in self.runs():
            d: Dict[str, tuple] = {}
            m = self.layers[r.layer].delta
            if m is not None:
                d["S"] = (m.heads, m.vdim, m.dim)
                d["conv"] = (m.conv_taps - 1,
                             2 * m.qk_heads * m.dim + m.heads * m.vdim)
            out.append(d)
        return out

    def cache_layout(self):
        from ..engine.kvcache import HybridStateLayout
        return HybridStateLayout(self._kv_shapes(), self.state_shapes())

    def state_bytes_per_seq(self) -> int:
        return self.cache_layout().state_bytes_per_seq()


def config_from_dict(d: dict, name: str = "mugazen") -> MugazenConfig:
    """MugazenConfig from a parsed config.json."""
    layers: List[MugazenLayerConfig] = []
    for i, ld in enumerate(d["layers"]):
        kind, mx = ld["type"], ld["mixer"]
        lc = MugazenLayerConfig(kind)
        if kind == "delta":
            lc.delta = MatrixMemoryConfig(
                ops.SCAN_DELTA_HEAD, heads=int(mx["heads"]),
                qk_heads=int(mx["kv_heads"]), dim=int(mx["dim"]),
                vdim=int(mx["vdim"]), conv_taps=int(mx["conv"]))
            if lc.delta.heads % lc.delta.qk_heads:
                raise ValueError(f"layer {i}: heads % kv_heads != 0")
            if lc.delta.conv_taps < 1:
                raise ValueError(f"layer {i}: conv must be >= 1")
        elif kind == "latent_attention":
            lc.latent = LatentMixerConfig(
                heads=int(mx["heads"]), dim=int(mx["dim"]),
                vdim=int(mx["vdim"]), q_rank=int(mx["q_rank"]),
                kv_rank=int(mx["kv_rank"]), window=CAUSAL_WINDOW,
                scale=float(mx["scale"]), gate="head", sink=True)
        else:
            raise ValueError(f"layer {i}: unsupported mixer {kind!r}")
        ml = ld.get("mlp")
        if ml is not None:
            if ml["kind"] == "dense":
                lc.mlp = MugazenFeedForwardConfig("dense", int(ml["ff"]),
                                                  limit=float(ml["limit"]))
            elif ml["kind"] == "moe":
                lc.mlp = MugazenFeedForwardConfig(
                    "moe", int(ml["expert"]["ff"]),
                    experts=int(ml["router"]["experts"]),
                    top=int(ml["router"]["top"]))
                if not 1 <= lc.mlp.top <= lc.mlp.experts:
                    raise ValueError(f"layer {i}: top out of range")
            else:
                raise ValueError(f"layer {i}: unsupported mlp {ml['kind']!r}")
        layers.append(lc)
    lp = d.get("loop") or {}
    cfg = MugazenConfig(
        name=name, vocab_size=int(d["vocab"]), hidden_size=int(d["width"]),
        layers=layers, norm_eps=float(d["norm"]["eps"]),
        embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
        max_positions=int(d["max_positions"]),
        loop_start=int(lp.get("start", 0)), loop_stop=int(lp.get("stop", 0)),
        loop_times=int(lp.get("times", 1)))
    if not 0 <= cfg.loop_start <= cfg.loop_stop <= len(layers):
        raise ValueError("loop.start .. loop.stop is not a range of layers")
    if cfg.loop_times < 1:
        raise ValueError("loop.times must be >= 1")
    return cfg


def config_from_checkpoint(path: str) -> MugazenConfig:
    with open(os.path.join(path, "config.json")) as f:
        return config_from_dict(json.load(f), name=path)


class ClampedFeedForward(GatedFeedForward):
    """down( g sigmoid(slope g) (u + 1) ), g = min(gate h, limit),
    u = clamp(up h, -limit, limit)."""

    def __init__(self, width: int, ff: int, limit: float, dtype):
        super().__init__(width, ff, "clamped", dtype)
        self.limit = limit

    def forward(self, h, allow_gather: bool = True):
        gu = ops.linear(h, self.gate_up)
        act = torch.empty(h.size(0), self.ff, dtype=h.dtype, device=h.device)
        ops.routed_clamped_glu(act, gu, None, 1, self.limit, UNIT_SLOPE)
        return ops.linear(act, self.down)


class TopSoftmaxExperts(GroupedSigmoidExperts):
    """SiLU-gated experts weighed by the softmax over the `top` largest
    router logits (biased), with no groups and no shared expert."""

    def __init__(self, width: int, fc: MugazenFeedForwardConfig, dtype):
        super().__init__(width, SipelornFeedForwardConfig(
            "moe", fc.ff, experts=fc.experts, top=fc.top), dtype)
        self.router = _param(fc.experts, width, dtype=dtype)

    def _route_params(self):
        self.router_bias = _param(self.fc.experts, dtype=torch.float32)

    @torch.no_grad()
    def _load_route(self, get):
        self.router.copy_(get("router"))
        self.router_bias.copy_(get("router.b").float())

    def route(self, h) -> torch.Tensor:
        logits = ops.narrow_linear(h, self.router, self.router_bias)
        weight = torch.empty_like(logits)
        return ops.grouped_softmax_route(weight, logits, None, self.fc.top,
                                         1, 1, 1.0)

    def forward(self, h, allow_gather: bool = True):
        return super().forward(h, allow_gather)[0]


class MugazenLayer(torch.nn.Module):
    def __init__(self, cfg: MugazenConfig, lc: MugazenLayerConfig, dtype):
        super().__init__()
        W = cfg.hidden_size
        f32 = torch.float32
        self.lc = lc
        self.norm1, self.norm1b = _param(W, dtype=f32), _param(W, dtype=f32)
        self.mix = (MatrixMemoryMixer(W, lc.delta, cfg.norm_eps, dtype)
                    if lc.delta is not None else
                    LatentAttention(W, lc.latent, cfg.norm_eps, dtype))
        if lc.mlp is None:
            self.mlp = None
        else:
            self.norm2, self.norm2b = (_param(W, dtype=f32),
                                       _param(W, dtype=f32))
            self.mlp = (ClampedFeedForward(W, lc.mlp.ff, lc.mlp.limit, dtype)
                        if lc.mlp.kind == "dense" else
                        TopSoftmaxExperts(W, lc.mlp, dtype))


class MugazenForCausalLM(torch.nn.Module):
    def __init__(self, cfg: MugazenConfig, device="cpu", tp_rank: int = 0,
                 tp_size: int = 1, seed: int = 0, dtype=torch.bfloat16):
        super().__init__()
        if tp_size != 1:
            raise ValueError("Mugazen: tensor parallelism is not implemented")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Mugazen: unsupported compute dtype {dtype}")
        self.cfg = cfg
        self.dtype = dtype
        self.tp_rank, self.tp_size, self.tp_group = 0, 1, None
        self.runs = cfg.runs()
        W = cfg.hidden_size
        f32 = torch.float32
        with torch.device(device):
            self.embed = _param(cfg.vocab_size, W, dtype=dtype)
            self.pos = _param(cfg.max_positions, W, dtype=dtype)
            self.embed_norm = _param(W, dtype=f32)
            self.loop_step = (_param(cfg.loop_times, W, dtype=f32)
                              if cfg.looped else None)
            self.layers = torch.nn.ModuleList(
                [MugazenLayer(cfg, lc, dtype) for lc in cfg.layers])
            self.final_norm = _param(W, dtype=f32)
            self.lm_head = _param(cfg.vocab_size, W, dtype=dtype)
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
            if leaf == "head_rate":
                normal(p, 0.5, -0.5)
            elif leaf == "gate_bias":
                normal(p, 0.5, -2.0)
            elif leaf in ("sink", "router_bias"):
                normal(p, 0.5)
            elif leaf in ("embed", "pos"):
                normal(p, 1.0)
            elif leaf == "loop_step":
                normal(p, 0.1)
            elif leaf == "w_conv":
                normal(p, 0.5)
            elif leaf == "w_uk":
                normal(p, 1.0 / p.size(1) ** 0.5)
            elif p.dim() >= 2:
                normal(p, 1.0 / p.size(-1) ** 0.5)
            else:
                p.fill_(1.0)
        for layer in self.layers:
            if layer.lc.latent is not None:    # keep the rank padding zero
                R = layer.lc.latent.kv_rank
                layer.mix.w_uk[:, :, R:] = 0
                layer.mix.w_uv[:, R:, :] = 0

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
        """Copy checkpoint tensors (embed, pos, embed.norm, loop.step,
        l<i>.norm1/1b/2/2b, l<i>.mix.*, l<i>.mlp.*, final.norm, head) into
        the fused serving layout."""
        dev, dt = self.embed.device, self.dtype

        def getter(prefix):
            def get(name):
                return sd[prefix + name].to(device=dev, dtype=dt)
            return get

        top = getter("")
        self.embed.copy_(top("embed"))
        self.pos.copy_(top("pos"))
        self.embed_norm.copy_(top("embed.norm").float())
        if self.loop_step is not None:
            self.loop_step.copy_(top("loop.step").float())
        self.final_norm.copy_(top("final.norm").float())
        self.lm_head.copy_(top("head"))
        for i, layer in enumerate(self.layers):
            g = getter(f"l{i}.")
            layer.norm1.copy_(g("norm1").float())
            layer.norm1b.copy_(g("norm1b").float())
            layer.mix.load(getter(f"l{i}.mix."))
            if layer.mlp is not None:
                layer.norm2.copy_(g("norm2").float())
                layer.norm2b.copy_(g("norm2b").float())
                layer.mlp.load(getter(f"l{i}.mlp."))

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor, md: AttnMetadata,
                kv_caches: List, last_rows: Optional[torch.Tensor] = None
                ) -> torch.Tensor:
        cfg, eps, W = self.cfg, self.cfg.norm_eps, self.cfg.hidden_size
        if md.state_slots is None:
            raise ValueError("Mugazen needs per-sequence state slots")
        T, dev = input_ids.size(0), input_ids.device
        f32 = torch.float32
        x = torch.empty(T, W, dtype=f32, device=dev)
        # what every pass but the first adds again
        x0 = torch.empty_like(x) if cfg.looped and cfg.loop_times > 1 else None
        ops.position_embed_norm(x, input_ids, md.positions, self.embed,
                                self.pos, cfg.embed_scale, self.embed_norm,
                                eps, x_copy=x0)

        def step(y, post, norm, run=None):
            """x += N(y; post) (y None: nothing), then what `run` takes in
            before its layer, then N(x; norm) for the next GEMM (norm None:
            nothing)."""
            out, rows, vec = None, None, None
            if norm is not None:
                out = torch.empty(T, W, dtype=self.dtype, device=dev)
            if run is not None and run.enters:
                vec = self.loop_step[run.loop_pass]
                rows = x0 if run.loop_pass > 0 else None
            ops.residual_update_norm(
                x, y, ops.UPDATE_NONE if y is None else ops.UPDATE_UNIT_RMS,
                None, None, post, eps, norm, None, out, rms_norm=True,
                add_rows=rows, add_vec=vec)
            return out

        trace = self.residual_trace
        n = len(self.runs)
        h = step(None, None, self.layers[self.runs[0].layer].norm1,
                 self.runs[0])
        for r, run in enumerate(self.runs):
            layer = self.layers[run.layer]
            pool, _none, state = kv_caches[r]
            if layer.lc.delta is not None:
                y = layer.mix(h, None, state, md)
            else:
                y = layer.mix(h, pool, md)
            post = layer.norm1b
            if layer.mlp is not None:
                h = step(y, post, layer.norm2)
                y = layer.mlp(h, allow_gather=md.is_prefill)
                post = layer.norm2b
            nxt = self.runs[r + 1] if r + 1 < n else None
            if nxt is not None:
                norm = self.layers[nxt.layer].norm1
            else:
                # only the wanted rows need the final norm
                norm = self.final_norm if last_rows is None else None
            if trace is not None:
                step(y, post, None)
                trace.append(x.clone())
                y = None
            h = step(y, post, norm, nxt)
        if last_rows is not None:
            x = x[last_rows]
            T = x.size(0)
            h = step(None, None, self.final_norm)
        return ops.linear(h, self.lm_head).float()


def _tiny(name: str) -> MugazenConfig:
    latent = LatentMixerConfig(
        heads=4, dim=32, vdim=32, q_rank=64, kv_rank=48,
        window=CAUSAL_WINDOW, scale=32 ** -0.5, gate="head", sink=True)
    delta = MatrixMemoryConfig(ops.SCAN_DELTA_HEAD, 4, 2, 32, 32, conv_taps=4)
    dense = MugazenFeedForwardConfig("dense", 256, limit=7.0)
    moe = MugazenFeedForwardConfig("moe", 64, experts=8, top=2)
    layers = [MugazenLayerConfig("delta", delta=delta, mlp=dense),
              MugazenLayerConfig("latent_attention", latent=latent, mlp=moe),
              MugazenLayerConfig("delta", delta=delta, mlp=moe)]
    return MugazenConfig(name=name, vocab_size=512, hidden_size=128,
                         layers=layers, norm_eps=1e-5, embed_scale=8.0,
                         max_positions=4096, loop_start=1, loop_stop=3,
                         loop_times=2)


MUGAZEN_CONFIGS: Dict[str, MugazenConfig] = {
    "tiny-mugazen": _tiny("tiny-mugazen"),
}


def make_mugazen_instance(name: str, device: str, engine_cfg,
                          weights_path: Optional[str] = None):
    """ModelInstance over a Mugazen model (engine factory hook): a named
    random-init config, or a checkpoint directory."""
    from ..engine.llm import ModelInstance

    cfg = (config_from_checkpoint(weights_path) if weights_path
           else MUGAZEN_CONFIGS[name])
    if device.startswith("cuda") and not (
            ops.gated_available() and ops.latent_available()
            and ops.recurrent_available()):
        raise RuntimeError(
            "GPU engine requires the gfx950 gated, latent and recurrent "
            "extensions (python -m agentainer_amd.ops.build gated latent "
            "recurrent)")
    return ModelInstance(name, cfg, device, engine_cfg,
                         weights_path=weights_path,
                         model_cls=MugazenForCausalLM)
