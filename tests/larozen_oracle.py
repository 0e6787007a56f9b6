"""Plain, slow float64 oracle for the Larozen design — one function per
mechanism, written from the design's equations and sharing no code with
the serving path (no cache manager, no state slots, no batching, no
kernels, no re-ordered weights). Whole sequences only.

Notation: x is the residual stream [T, W]; linear weights are stored
[out, in] and applied as y = W x; p counts positions from 0; w maps tensor
names to float64 tensors; U(v) = v / sqrt(mean(v^2) + eps).

  embedding   e_p = embed[tok_p]; the same table maps the last norm's output
              to logits
  layer       x += mixer(U(x) (1 + n1));  x += ff(U(x) (1 + n2))
  loop        layers start..stop-1 run `times` times with shared weights and
              separate memories; every pass starts with x <- W_in [x; e]
  mixers      "attention": values are the projected keys themselves, rotary
              on neighbouring pairs of the leading coordinates, capped
              scores; "parallel": an attention without positions (q and k
              normed over all heads together, a query factor that grows
              with the position, a sink in the softmax) beside a state-space
              recurrence with one decay per head (short convolution, step
              sizes, a skip, gate before a grouped norm), summed half and
              half after a norm each
  ff          down( max(up h, 0)^2 )
"""

from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional

import torch

F64 = torch.float64


# ----------------------------------------------------------------- pieces

def unit_rms(v, eps):
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def layer_norm_one_plus(x, weight, eps):
    return unit_rms(x, eps) * (1.0 + weight)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def rotate_neighbours(u, dims: int, base: float):
    """u [T, heads, D]: coordinates (2i, 2i+1), i < dims/2, turn by the angle
    p * base^(-2i/dims); the others pass."""
    out = u.clone()
    for p in range(u.shape[0]):
        for i in range(dims // 2):
            a = p * base ** (-2.0 * i / dims)
            c, s = math.cos(a), math.sin(a)
            x, y = u[p, :, 2 * i], u[p, :, 2 * i + 1]
            out[p, :, 2 * i] = x * c - y * s
            out[p, :, 2 * i + 1] = y * c + x * s
    return out


def softmax_attention(q, k, v, scale, cap=None, sink=None):
    """q [T, H, D]; k [T, G, D]; v [T, G, Dv]; causal; query head h reads
    key/value head h // (H/G). cap: scores become cap tanh(score / cap);
    sink [H]: exp(sink_h) joins head h's denominator once."""
    T, H = q.shape[:2]
    share = H // k.shape[1]
    o = torch.zeros(T, H, v.shape[2], dtype=v.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // share].T) * scale
        if cap is not None:
            s = cap * torch.tanh(s / cap)
        for i in range(T):
            row = s[i, :i + 1]
            top = row.max()
            if sink is not None:
                top = torch.maximum(top, sink[h])
            e = torch.exp(row - top)
            den = e.sum()
            if sink is not None:
                den = den + torch.exp(sink[h] - top)
            o[i, h] = (e @ v[:i + 1, h // share]) / den
    return o


def query_factor(T: int, coef: float, every: int):
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1.0)
                         for p in range(T)], dtype=F64)


def short_convolution(u, kernel, bias):
    """u [T, C], kernel [C, taps], the last column weighs the current row;
    rows before the sequence are zero."""
    T, taps = u.shape[0], kernel.shape[1]
    y = bias.expand_as(u).clone()
    for back in range(taps):
        if back < T:
            y[back:] += kernel[:, taps - 1 - back] * u[:T - back]
    return y


def state_space_recurrence(x, B, C, step, rate, skip):
    """x [T, H, Dv]; B, C [T, G, N]; step [T, H]; rate, skip [H]. The memory
    S [N, Dv] decays by exp(-rate step), takes in step B x^T and is read by
    C afterwards; the skip adds the token's own x."""
    T, H, Dv = x.shape
    share = H // B.shape[1]
    y = torch.zeros_like(x)
    for h in range(H):
        S = torch.zeros(B.shape[2], Dv, dtype=x.dtype)
        for t in range(T):
            b, c = B[t, h // share], C[t, h // share]
            S = torch.exp(-rate[h] * step[t, h]) * S \
                + step[t, h] * torch.outer(b, x[t, h])
            y[t, h] = c @ S + skip[h] * x[t, h]
    return y


def gate_then_group_norm(y, z, weight, parts: int, eps):
    """y, z [T, inner]: y silu(z), every one of `parts` equal consecutive
    parts brought to unit rms on its own, then one weight vector."""
    g = y * silu(z)
    return unit_rms(g.view(g.shape[0], parts, -1), eps).reshape(g.shape) \
        * weight


# ----------------------------------------------------------------- mixers

def linear(h, w, name):
    y = h @ w[name].T
    return y + w[name + ".b"] if name + ".b" in w else y


def shared_kv_mixer(h, w, p, mx, eps):
    T = h.shape[0]
    H, G, D = mx["heads"], mx["kv_heads"], mx["dim"]
    q = linear(h, w, p + "q").view(T, H, D)
    k = linear(h, w, p + "k").view(T, G, D)
    rot = mx["rot"]
    o = softmax_attention(
        rotate_neighbours(q, rot["dims"], rot["base"]),
        rotate_neighbours(k, rot["dims"], rot["base"]), k,
        float(mx["scale"]), cap=float(mx["softcap"]))
    return o.reshape(T, H * D) @ w[p + "o"].T


def positionless_mixer(h, w, p, mx, eps):
    T = h.shape[0]
    H, G = mx["heads"], mx["kv_heads"]
    q = unit_rms(linear(h, w, p + "q"), eps) * w[p + "q.norm"]
    k = unit_rms(linear(h, w, p + "k"), eps) * w[p + "k.norm"]
    v = linear(h, w, p + "v")
    t = mx["q_temp"]
    q = q * query_factor(T, float(t["coef"]), t["every"]).unsqueeze(1)
    o = softmax_attention(q.view(T, H, mx["dim"]), k.view(T, G, mx["dim"]),
                          v.view(T, G, mx["vdim"]), float(mx["scale"]),
                          sink=w[p + "sink"])
    return linear(o.reshape(T, H * mx["vdim"]), w, p + "o")


def state_space_mixer(h, w, p, mx, eps):
    T = h.shape[0]
    H, Dv, N, G = mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = H * Dv
    z, xbc, dt = torch.split(h @ w[p + "in"].T,
                             [inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(short_convolution(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=1)
    y = state_space_recurrence(
        x.reshape(T, H, Dv), B.reshape(T, G, N), C.reshape(T, G, N),
        softplus(dt + w[p + "dt_bias"]), torch.exp(w[p + "A_log"]),
        w[p + "D"])
    y = gate_then_group_norm(y.reshape(T, inner), z, w[p + "norm"],
                             mx["norm_groups"], eps)
    return y @ w[p + "o"].T


def parallel_mixer(h, w, p, mx, eps):
    a = positionless_mixer(h, w, p + "left.", mx["left"], eps)
    b = state_space_mixer(h, w, p + "right.", mx["right"], eps)
    return 0.5 * (unit_rms(a, eps) * w[p + "left.out"]
                  + unit_rms(b, eps) * w[p + "right.out"])


def squared_relu_ff(h, w, p):
    return torch.clamp(h @ w[p + "up"].T, min=0.0) ** 2 @ w[p + "down"].T


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
    e0 = w["embed"][torch.tensor(tokens)]
    x = e0
    for i, t in run_order(cfg):
        layer, L = cfg["layers"][i], f"l{i}."
        if t is not None and i == cfg["loop"]["start"]:
            x = torch.cat([x, e0], dim=1) @ w["loop.in"].T
        mix = {"attention": shared_kv_mixer,
               "parallel": parallel_mixer}[layer["type"]]
        x = x + mix(layer_norm_one_plus(x, w[L + "norm1"], eps), w,
                    L + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + squared_relu_ff(
                layer_norm_one_plus(x, w[L + "norm2"], eps), w, L + "mlp.")
        if trace is not None:
            trace.append(x.clone())
    return layer_norm_one_plus(x, w["final.norm"], eps) @ w["embed"].T


# ----------------------------------------------- small random checkpoints

def attention_layer(heads=4, kv_heads=2, dim=16, rot_dims=8, base=500.0,
                    scale=None, softcap=6.0):
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
        "rot": {"base": base, "dims": rot_dims}, "softcap": softcap,
        "scale": scale if scale is not None else dim ** -0.5}}


def left_mixer(heads=6, kv_heads=2, dim=16, vdim=12, coef=0.4, every=5,
               scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": scale if scale is not None else dim ** -0.5,
            "q_temp": {"coef": coef, "every": every}}


def right_mixer(heads=4, vdim=12, state=20, groups=2, conv=3, norm_groups=3):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
            "conv": conv, "norm_groups": norm_groups}


def parallel_layer(left=None, right=None):
    return {"type": "parallel", "mixer": {"left": left or left_mixer(),
                                          "right": right or right_mixer()}}


def make_config(layers, vocab=96, width=48, eps=1e-5, loop=None) -> dict:
    """layers: [(mixer dict from attention_layer / parallel_layer, inner
    size of the feed-forward or None)]; loop: (start, stop, times) or
    None."""
    cfg = {"architecture": "Larozen", "vocab": vocab, "width": width,
           "norm": {"eps": eps},
           "layers": [dict(m, mlp=None if ff is None else
                           {"kind": "dense", "ff": ff}) for m, ff in layers]}
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

    w = {"embed": mat(V, W, math.sqrt(W) * 0.8), "final.norm": vec(W)}
    if cfg.get("loop"):
        w["loop.in"] = mat(W, 2 * W, 1.2)
    for i, layer in enumerate(cfg["layers"]):
        L, p, mx = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        w[L + "norm1"] = vec(W)
        if layer["type"] == "attention":
            H, G, D = mx["heads"], mx["kv_heads"], mx["dim"]
            for nm, n in (("q", H * D), ("k", G * D)):
                w[p + nm] = mat(n, W, 1.5)
                w[p + nm + ".b"] = vec(n, 0.0, 0.5)
            w[p + "o"] = mat(W, H * D)
        else:
            a, r = mx["left"], mx["right"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for nm, n in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                w[p + "left." + nm] = mat(n, W)
                w[p + f"left.{nm}.b"] = vec(n, 0.0, 0.5)
            w[p + "left.q.norm"] = vec(H * D, 1.3, 0.3)
            w[p + "left.k.norm"] = vec(G * D, 1.3, 0.3)
            w[p + "left.sink"] = vec(H, 1.0, 0.8)
            w[p + "left.o"] = mat(W, H * Dv)
            w[p + "left.o.b"] = vec(W, 0.0, 0.5)
            H, Dv, N, G = r["heads"], r["vdim"], r["state"], r["groups"]
            inner, C = H * Dv, H * Dv + 2 * G * N
            w[p + "right.in"] = mat(inner + C + H, W, 1.5)
            w[p + "right.conv"] = (torch.randn(C, r["conv"], generator=g)
                                   * 0.6).bfloat16().float()
            w[p + "right.conv.b"] = vec(C, 0.0, 0.4)
            w[p + "right.dt_bias"] = vec(H, -1.5, 0.7)
            w[p + "right.A_log"] = vec(H, -0.5, 0.7)
            w[p + "right.D"] = vec(H, 0.7, 0.4)
            w[p + "right.norm"] = vec(inner, 1.0, 0.2)
            w[p + "right.o"] = mat(W, inner)
            w[p + "left.out"] = vec(W, 1.0, 0.2)
            w[p + "right.out"] = vec(W, 1.0, 0.2)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            w[L + "norm2"] = vec(W)
            w[L + "mlp.up"] = mat(ff, W)
            w[L + "mlp.down"] = mat(W, ff)
    return w


def save_checkpoint(path: str, cfg: dict, weights: Dict[str, torch.Tensor]):
    """Write config.json + model.safetensors (bf16) into `path`."""
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in weights.items()},
              os.path.join(path, "model.safetensors"))
