"""Plain, slow float64 oracle for the Mugazen design — one function per
mechanism, written from the design's equations and sharing no code with
the serving path (no cache manager, no state slots, no batching, no
kernels, no absorbed weights). Whole sequences only.

Notation: x is the residual stream [T, W]; linear weights are stored
[out, in] and applied as y = W x; p counts positions from 0; w maps tensor
names to float64 tensors; N(v; a) = v / sqrt(mean(v^2) + eps) * a.

  embedding   e_p = N(scale * embed[tok_p] + pos[p]; embed.norm)
  layer       x += N(mixer(N(x; n1)); n1b);  x += N(ff(N(x; n2)); n2b)
  loop        layers start..stop-1 run `times` times with shared weights and
              separate memories; pass t starts with
              x += [t > 0] e + loop.step[t]
  mixers      "delta": gated delta rule over a matrix memory, one decay and
              one write strength per head; "latent_attention": keys and
              values expanded from an RMS-normed latent, queries through a
              latent of their own, a sink in the softmax, one sigmoid gate
              per head.
  ff          clamped dense unit, or softmax-of-top-k routed SiLU experts.
"""

from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional

import torch

F64 = torch.float64
CLAMP_SLOPE = 1.702
UNIT_EPS = 1e-6


# ----------------------------------------------------------------- pieces

def rms_norm(v, weight, eps):
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps) * weight


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def unit_vector(v):
    return v / torch.sqrt((v * v).sum(dim=-1, keepdim=True) + UNIT_EPS)


def embed_tokens(tokens: List[int], w, scale: float, eps: float):
    T = len(tokens)
    x = w["embed"][torch.tensor(tokens)] * scale + w["pos"][:T]
    return rms_norm(x, w["embed.norm"], eps)


def short_convolution(u, kernel):
    """u [T, C], kernel [C, taps], the last column weighs the current row;
    rows before the sequence are zero."""
    T, taps = u.shape[0], kernel.shape[1]
    y = torch.zeros_like(u)
    for back in range(taps):
        if back < T:
            y[back:] += kernel[:, taps - 1 - back] * u[:T - back]
    return y


# ----------------------------------------------------------------- mixers

def delta_recurrence(q, k, v, decay, beta):
    """q, k [T, G, D]; v [T, H, Dv]; decay, beta [T, H] -> o [T, H, Dv].
    The memory is decayed, then corrected towards v, then read."""
    T, H, Dv = v.shape
    share = H // k.shape[1]
    o = torch.zeros(T, H, Dv, dtype=v.dtype)
    for h in range(H):
        S = torch.zeros(k.shape[2], Dv, dtype=v.dtype)
        for t in range(T):
            kt, qt = k[t, h // share], q[t, h // share]
            S = decay[t, h] * S
            u = beta[t, h] * (v[t, h] - kt @ S)
            S = S + torch.outer(kt, u)
            o[t, h] = qt @ S
    return o


def delta_decay(pre, a_log, dt_bias):
    return torch.exp(-torch.exp(a_log) * softplus(pre + dt_bias))


def delta_mixer(h, w, p, mx, eps):
    T = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]

    def branch(name, heads):
        u = short_convolution(h @ w[p + name].T, w[p + name + ".conv"])
        return silu(u).view(T, heads, -1)

    q = unit_vector(branch("q", G)) * D ** -0.5
    k = unit_vector(branch("k", G))
    v = branch("v", H)
    beta = sigmoid(h @ w[p + "b"].T)
    decay = delta_decay(h @ w[p + "a"].T, w[p + "A_log"], w[p + "dt_bias"])
    o = delta_recurrence(q, k, v, decay, beta)
    o = rms_norm(o, w[p + "norm"], eps)
    gate = silu(h @ w[p + "g"].T).view(T, H, Dv)
    return (o * gate).reshape(T, H * Dv) @ w[p + "o"].T


def sink_softmax_attention(q, k, v, scale, sink):
    """q, k [T, H, D]; v [T, H, Dv]; causal; exp(sink_h) joins the
    denominator of head h once."""
    T, H = q.shape[:2]
    o = torch.zeros(T, H, v.shape[2], dtype=v.dtype)
    for i in range(T):
        for h in range(H):
            s = (k[:i + 1, h] @ q[i, h]) * scale
            top = max(float(s.max()), float(sink[h]))
            e = torch.exp(s - top)
            o[i, h] = (e @ v[:i + 1, h]) / (e.sum()
                                            + math.exp(float(sink[h]) - top))
    return o


def latent_mixer(h, w, p, mx, eps):
    T = h.shape[0]
    H, D, Dv = mx["heads"], mx["dim"], mx["vdim"]
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    c = rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)
    q = (cq @ w[p + "uq"].T).view(T, H, D)
    k = (c @ w[p + "uk"].T).view(T, H, D)
    v = (c @ w[p + "uv"].T).view(T, H, Dv)
    o = sink_softmax_attention(q, k, v, float(mx["scale"]), w[p + "sink"])
    o = o * sigmoid(h @ w[p + "g"].T).unsqueeze(-1)
    return o.reshape(T, H * Dv) @ w[p + "o"].T


# ----------------------------------------------------------- feed-forward

def clamped_unit(gate, up, limit):
    g = torch.clamp(gate, max=limit)
    u = torch.clamp(up, min=-limit, max=limit)
    return g * sigmoid(CLAMP_SLOPE * g) * (u + 1.0)


def dense_ff(h, w, p, ml):
    return clamped_unit(h @ w[p + "gate"].T, h @ w[p + "up"].T,
                        float(ml["limit"])) @ w[p + "down"].T


def route(h, w, p, r):
    """Per token [(expert, weight)]: the `top` largest logits, softmax over
    those only."""
    z = h @ w[p + "router"].T + w[p + "router.b"]
    out = []
    for row in z.tolist():
        best = sorted(range(len(row)), key=lambda e: -row[e])[:r["top"]]
        m = max(row[e] for e in best)
        ex = [math.exp(row[e] - m) for e in best]
        out.append([(e, x / sum(ex)) for e, x in zip(best, ex)])
    return out


def expert_mixture(h, w, p, ml):
    y = torch.zeros_like(h)
    for t, chosen in enumerate(route(h, w, p, ml["router"])):
        for e, wt in chosen:
            a = silu(w[f"{p}e{e}.gate"] @ h[t]) * (w[f"{p}e{e}.up"] @ h[t])
            y[t] += wt * (w[f"{p}e{e}.down"] @ a)
    return y


# ---------------------------------------------------------------- forward

def run_order(cfg) -> List[tuple]:
    """(layer, pass or None): the order in which layers run; pass is None
    outside the loop."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    return ([(i, None) for i in range(a)]
            + [(i, t) for t in range(lp["times"]) for i in range(a, b)]
            + [(i, None) for i in range(b, n)])


def forward(tokens: List[int], weights: Dict[str, torch.Tensor], cfg: dict,
            trace: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence; `trace` (a list) receives the
    residual stream after every layer run."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    e0 = embed_tokens(tokens, w, float(cfg["embedding"]["scale"]), eps)
    x = e0
    for i, t in run_order(cfg):
        layer, L = cfg["layers"][i], f"l{i}."
        if t is not None and i == cfg["loop"]["start"]:
            x = x + w["loop.step"][t] + (e0 if t > 0 else 0.0)
        mix = {"delta": delta_mixer,
               "latent_attention": latent_mixer}[layer["type"]]
        y = mix(rms_norm(x, w[L + "norm1"], eps), w, L + "mix.",
                layer["mixer"], eps)
        x = x + rms_norm(y, w[L + "norm1b"], eps)
        ml = layer.get("mlp")
        if ml is not None:
            ff = dense_ff if ml["kind"] == "dense" else expert_mixture
            y = ff(rms_norm(x, w[L + "norm2"], eps), w, L + "mlp.", ml)
            x = x + rms_norm(y, w[L + "norm2b"], eps)
        if trace is not None:
            trace.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


# ----------------------------------------------- small random checkpoints

def delta_layer(heads=4, kv_heads=2, dim=16, vdim=12, conv=3):
    return {"type": "delta", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "conv": conv}}


def latent_layer(heads=3, dim=16, vdim=12, q_rank=20, kv_rank=24, scale=None):
    return {"type": "latent_attention", "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank,
        "kv_rank": kv_rank,
        "scale": scale if scale is not None else dim ** -0.5}}


def dense_mlp(ff=48, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe_mlp(experts=6, top=2, ff=20):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top}}


def make_config(layers, vocab=96, width=48, eps=1e-5, embed_scale=3.0,
                max_positions=192, loop=None) -> dict:
    """layers: [(mixer dict from delta_layer/latent_layer, mlp dict or
    None)]; loop: (start, stop, times) or None."""
    cfg = {"architecture": "Mugazen", "vocab": vocab, "width": width,
           "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
           "max_positions": max_positions,
           "layers": [dict(m, mlp=ml) for m, ml in layers]}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """Random weights (values representable in bf16) for a config dict."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def mat(rows, cols, gain=1.0):
        return (torch.randn(rows, cols, generator=g) * gain / math.sqrt(cols)
                ).bfloat16().float()

    def vec(n, mean=0.0, std=0.1):
        return (mean + torch.randn(n, generator=g) * std).bfloat16().float()

    w = {"embed": mat(V, W, math.sqrt(W) * 0.4), "head": mat(V, W),
         "pos": mat(cfg["max_positions"], W, math.sqrt(W) * 0.6),
         "embed.norm": vec(W, 1.0), "final.norm": vec(W, 1.0)}
    if cfg.get("loop"):
        w["loop.step"] = mat(cfg["loop"]["times"], W, math.sqrt(W) * 0.4)
    for i, layer in enumerate(cfg["layers"]):
        L, p, mx = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        w[L + "norm1"] = vec(W, 1.0)
        w[L + "norm1b"] = vec(W, 0.7, 0.2)
        H, D, Dv = mx["heads"], mx["dim"], mx["vdim"]
        if layer["type"] == "delta":
            G = mx["kv_heads"]
            for nm, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                w[p + nm] = mat(rows, W, 2.0)
                w[p + nm + ".conv"] = (torch.randn(rows, mx["conv"],
                                                   generator=g) * 0.6
                                       ).bfloat16().float()
            w[p + "b"] = mat(H, W, 1.5)
            w[p + "a"] = mat(H, W, 1.5)
            w[p + "A_log"] = vec(H, -0.5, 0.7)
            w[p + "dt_bias"] = vec(H, -2.0, 0.7)
            w[p + "norm"] = vec(Dv, 1.0)
            w[p + "g"] = mat(H * Dv, W, 1.5)
        else:
            R, Rq = mx["kv_rank"], mx["q_rank"]
            w[p + "dq"] = mat(Rq, W)
            w[p + "dq.norm"] = vec(Rq, 1.0)
            w[p + "uq"] = mat(H * D, Rq, 2.0)
            w[p + "dkv"] = mat(R, W)
            w[p + "dkv.norm"] = vec(R, 1.0)
            w[p + "uk"] = mat(H * D, R, 1.5)
            w[p + "uv"] = mat(H * Dv, R)
            w[p + "sink"] = vec(H, 1.0, 0.8)
            w[p + "g"] = mat(H, W, 1.5)
        w[p + "o"] = mat(W, H * Dv)
        ml = layer.get("mlp")
        if ml is None:
            continue
        q = L + "mlp."
        w[L + "norm2"] = vec(W, 1.0)
        w[L + "norm2b"] = vec(W, 0.7, 0.2)
        if ml["kind"] == "dense":
            w[q + "gate"] = mat(ml["ff"], W, 1.5)
            w[q + "up"] = mat(ml["ff"], W, 1.5)
            w[q + "down"] = mat(W, ml["ff"])
        else:
            E, Fe = ml["router"]["experts"], ml["expert"]["ff"]
            # wide logits: choices do not sit on rounding-sized margins
            w[q + "router"] = mat(E, W, 3.0)
            w[q + "router.b"] = vec(E, 0.0, 1.0)
            for e in range(E):
                w[f"{q}e{e}.gate"] = mat(Fe, W, 2.0)
                w[f"{q}e{e}.up"] = mat(Fe, W, 2.0)
                w[f"{q}e{e}.down"] = mat(W, Fe)
    return w


def save_checkpoint(path: str, cfg: dict, weights: Dict[str, torch.Tensor]):
    """Write config.json + model.safetensors (bf16) into `path`."""
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in weights.items()},
              os.path.join(path, "model.safetensors"))
