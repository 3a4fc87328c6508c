"""Plain, slow implementation of the Fumanex decoder: whole sequences, no cache, one function
for each mechanism, float64 arithmetic on the CPU.  It shares no code with the engine under
``zinfer_amd/``: it is the oracle the engine is compared with.

The design in this file's own notation (x: the residual stream of one sequence, [T, W];
p: a token's position, counted from 0; h: what both sublayers of a layer read):

  x_p        = E[token_p] * c
  layer:       h = N(x);  x <- x + (mix(h) + ff(h))              one norm, two readers
  N(v)       = v / sqrt(mean v^2 + eps) * w;   u(v) = v / sqrt(mean v^2 + eps)
  'attention': q = Wq h + bq, k = Wk h + bk, v = Wv h + bv;  q <- u(q), k <- u(k) a head
               s_ij = t * tanh(scale * q_i . k_j / t) + rel[bucket(i - j), head]
               j is seen by i:  j <= i and (i - j < size or j < keep)
               a_ij = exp s_ij / (exp sink_head + sum_j exp s_ij);  o_i = sum_j a_ij v_j
               layers that mix values: the first keeps its own v as v1, every later one takes
               v <- (1 - lam) v + lam v1, token by token
               mix = Wo o + bo
  bucket(n)  = n below B/2, then B/2 + floor(ln(n / (B/2)) / ln(D / (B/2)) * (B - B/2)), at
               most B - 1
  'retention': q, k = R_p(Wq h), R_p(Wk h) d^(-1/2), v = Wv h;  R_p turns the pairs (i, i + r/2)
               of a head's first r elements by p b^(-2i/r)
               S_t = g S_(t-1) + k_t v_t^T, o_t = S_t^T q_t        g: one number a head
               mix = Wo (u(o) a head * silu(Wg h))
  'lightning': q, k, v = silu(Wq h), silu(Wk h), silu(Wv h), the same S and o
               mix = Wo (N(o over all heads together) * sigmoid(Wg h))
  ff:          Wd gelu(Wu h + bu) + bd                              gelu: the tanh form
  logits     = H N_final(x) * logit_scale
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence

import torch

F64 = torch.float64


# ----------------------------------------------------------------------------- small pieces
def unit_rms(v: torch.Tensor, eps: float) -> torch.Tensor:
    """v over its root mean square, along the last dimension."""
    v = v.to(F64)
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def rms_norm(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(v, eps) * w.to(F64)


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def linear(w: torch.Tensor, h: torch.Tensor, b: Optional[torch.Tensor] = None) -> torch.Tensor:
    """W stored [out, in], applied to every row of h, a bias added."""
    y = h.to(F64) @ w.to(F64).T
    return y if b is None else y + b.to(F64)


# ----------------------------------------------------------------------------- attention
def bucket(n: int, buckets: int, far: float) -> int:
    """The row of the distance table for a key n positions back."""
    near = buckets // 2
    if n < near:
        return n
    grown = math.log(n / near) / math.log(far / near) * (buckets - near)
    # (a logarithm's last bit must not move a distance that lies on a bucket's edge)
    return min(buckets - 1, near + math.floor(grown + 1e-9))


def distance_bias(table: torch.Tensor, T: int, far: float) -> torch.Tensor:
    """[heads, T, T]: entry (h, i, j) is the table's number for the distance i - j (j <= i)."""
    B, H = table.shape
    rows = torch.tensor([bucket(n, B, far) for n in range(T)], dtype=torch.long)
    by_distance = table.to(F64)[rows]                            # [T, H]
    i = torch.arange(T)
    n = (i[:, None] - i[None, :]).clamp(min=0)
    return by_distance[n].permute(2, 0, 1)


def seen(T: int, size: Optional[int], keep: int) -> torch.Tensor:
    """[T, T] bool: whether position i sees position j."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if size is not None:
        ok = ok & ((i - j < size) | (j < keep))
    return ok


def sink_softmax(scores: torch.Tensor, visible: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """scores [H, T, T], sink [H]: weights whose denominator holds exp(sink) once more."""
    s = scores.masked_fill(~visible, -math.inf)
    column = sink.to(F64)[:, None, None].expand(s.shape[0], s.shape[1], 1)
    both = torch.cat([column, s], dim=-1)
    both = torch.exp(both - both.max(dim=-1, keepdim=True).values)
    return (both / both.sum(dim=-1, keepdim=True))[..., 1:]


def attention_values(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict) -> torch.Tensor:
    G, dv = int(m["kv_heads"]), int(m["vdim"])
    return linear(w["v"], h, w["v.b"]).view(h.shape[0], G, dv)


def mixed_values(v: torch.Tensor, first: torch.Tensor, lam: float) -> torch.Tensor:
    return (1.0 - lam) * v + lam * first


def attention_scores(q, k, m: dict, table) -> torch.Tensor:
    """[H, T, T] from q [T, H, d] and k [T, G, d], capped, with the distance's bias."""
    T, H, _ = q.shape
    kk = k.repeat_interleave(H // k.shape[1], dim=1)
    s = torch.matmul(q.permute(1, 0, 2), kk.permute(1, 2, 0)) * float(m["scale"])
    cap = m.get("softcap")
    if cap is not None:
        s = float(cap) * torch.tanh(s / float(cap))
    return s + distance_bias(table, T, float(m["bias_max"]))


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float,
                    first_values: Optional[torch.Tensor]) -> torch.Tensor:
    """``first_values`` [T, G, dv]: the values of the first layer that mixes them (None: this
    layer takes its own as they are)."""
    H, G, d, dv = (int(m[n]) for n in ("heads", "kv_heads", "dim", "vdim"))
    h = h.to(F64)
    T = h.shape[0]
    q = unit_rms(linear(w["q"], h, w["q.b"]).view(T, H, d), eps)
    k = unit_rms(linear(w["k"], h, w["k.b"]).view(T, G, d), eps)
    v = attention_values(h, w, m)
    if first_values is not None:
        v = mixed_values(v, first_values, float(w["vmix"]))
    mask = m.get("mask") or {}
    a = sink_softmax(attention_scores(q, k, m, w["rel"]),
                     seen(T, mask.get("size"), int(mask.get("keep_first", 0))), w["sink"])
    o = torch.matmul(a, v.repeat_interleave(H // G, dim=1).permute(1, 0, 2))      # [H, T, dv]
    return linear(w["o"], o.permute(1, 0, 2).reshape(T, H * dv), w["o.b"])


# ----------------------------------------------------------------------------- recurrences
def rotate(z: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """z [T, heads, d]: the pairs (i, i + dims/2) of the first ``dims`` elements turned."""
    out = z.to(F64).clone()
    half = dims // 2
    for i in range(half):
        a = positions.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = z[:, :, i].to(F64), z[:, :, i + half].to(F64)
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def decayed_sums(q, k, v, decay: Sequence[float], state=None):
    """q, k [T, H, d], v [T, H, dv], one decay a head.  Returns (o [T, H, dv], S [H, d, dv])."""
    T, H, d = q.shape
    g = torch.tensor([float(x) for x in decay], dtype=F64)[:, None, None]
    S = torch.zeros((H, d, v.shape[2]), dtype=F64) if state is None else state.to(F64).clone()
    o = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for t in range(T):
        S = g * S + k[t].to(F64)[:, :, None] * v[t].to(F64)[:, None, :]
        o[t] = (q[t].to(F64)[:, :, None] * S).sum(dim=1)
    return o, S


def retention_mixer(h, w, m: dict, eps: float) -> torch.Tensor:
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    h = h.to(F64)
    T = h.shape[0]
    p = torch.arange(T)
    q, k = linear(w["q"], h).view(T, H, d), linear(w["k"], h).view(T, H, d)
    if m.get("rot") is not None:
        dims, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
        q, k = rotate(q, p, dims, base), rotate(k, p, dims, base)
    k = k * d ** -0.5
    o, _ = decayed_sums(q, k, linear(w["v"], h).view(T, H, dv), m["decay"])
    o = unit_rms(o, eps).reshape(T, H * dv)
    return linear(w["o"], o * silu(linear(w["g"], h)))


def lightning_mixer(h, w, m: dict, eps: float) -> torch.Tensor:
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    h = h.to(F64)
    T = h.shape[0]
    q, k = (silu(linear(w[n], h)).view(T, H, d) for n in "qk")
    o, _ = decayed_sums(q, k, silu(linear(w["v"], h)).view(T, H, dv), m["decay"])
    o = rms_norm(o.reshape(T, H * dv), w["norm"], eps)
    return linear(w["o"], o * sigmoid(linear(w["g"], h)))


# ----------------------------------------------------------------------------- the model
def feed_forward(h, w) -> torch.Tensor:
    return linear(w["down"], gelu_tanh(linear(w["up"], h, w["up.b"])), w["down.b"])


def below(tensors: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {n[len(prefix):]: t for n, t in tensors.items() if n.startswith(prefix)}


def layer(i: int, x: torch.Tensor, config: dict, tensors, shared: dict) -> torch.Tensor:
    """The stream after layer i.  ``shared["values"]``: what the first layer that mixes values
    leaves for the later ones (this function puts it there)."""
    L = config["layers"][i]
    eps = float(config["norm"]["eps"])
    h = rms_norm(x, tensors[f"l{i}.norm1"], eps)
    w, m = below(tensors, f"l{i}.mix."), L["mixer"]
    if L["type"] == "attention":
        first = None
        if m.get("v_mix"):
            first = shared.get("values")
            if first is None:
                shared["values"] = attention_values(h, w, m)
        y = attention_mixer(h, w, m, eps, first)
    elif L["type"] == "retention":
        y = retention_mixer(h, w, m, eps)
    else:
        y = lightning_mixer(h, w, m, eps)
    if L.get("mlp") is not None:
        y = y + feed_forward(h, below(tensors, f"l{i}.mlp."))
    return x + y


def embedding(token_ids: Sequence[int], config: dict, tensors) -> torch.Tensor:
    ids = torch.tensor(list(token_ids), dtype=torch.long)
    scale = (config.get("embedding") or {}).get("scale", 1.0)
    return tensors["embed"].to(F64)[ids] * float(scale)


def forward(token_ids: Sequence[int], config: dict, tensors,
            after_layers: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; ``after_layers`` takes the stream after every
    layer."""
    x = embedding(token_ids, config, tensors)
    shared: dict = {}
    for i in range(len(config["layers"])):
        x = layer(i, x, config, tensors, shared)
        if after_layers is not None:
            after_layers.append(x.clone())
    x = rms_norm(x, tensors["final.norm"], float(config["norm"]["eps"]))
    return linear(tensors["head"], x) * float(config.get("logit_scale") or 1.0)


def greedy(prompt: Sequence[int], n: int, config: dict, tensors) -> List[int]:
    out = list(prompt)
    for _ in range(n):
        out.append(int(torch.argmax(forward(out, config, tensors)[-1])))
    return out[len(prompt):]
