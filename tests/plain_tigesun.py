"""Plain, slow implementation of the Tigesun decoder: whole sequences, no cache, one function for
each mechanism, float64 arithmetic on the CPU.  It shares no code with the engine under
``zinfer_amd/``: it is the oracle the engine is compared with.

The design in this file's own notation (x: the residual stream of one sequence, [T, W]; p: a
token's position, counted from 0; N_w(v) = w v / sqrt(mean v^2 + eps)):

  x_p          = N_e(E[token_p])
  layer:         x <- x + N_b(mix(N_a(x)));   x <- x + N_d(ff(N_c(x)))   (the second only with an ff)
  'attention':   q, k, v = Wq h, Wk h, Wv h;   q, k <- R_p(N(q)), R_p(N(k)) a head (one gain each)
                 a_ij = softmax_j<=i (scale q_i . k_j);  o_i = sum_j a_ij v_j;  mix = Wo o
                 R_p turns the pairs (i, i + r/2) of a head's first r elements by p f_i (the
                 frequencies stretched by ``stretched``) and lengthens them
  'latent_attention':  c = N(Wc h);  k = Uk c, v = Uv c a head;  q = Wq h;  the same soft-max over
                 the last ``size`` positions, no rotation
  'mamba2':      Wi h = [z | x | B | C | s];  x, B, C <- silu(conv + b) a channel;
                 dt = softplus(s + b_dt);  S_t = exp(-exp(A) dt) S_(t-1) + dt B_t x_t^T a head,
                 y_t = S_t^T C_t + D x_t  (neighbouring heads share B and C);
                 u = y silu(z);  mix = Wo (u normed in equal parts, times a gain)
  ff:            Wd (gelu(Wg h + bg) (Wu h + bu)) + bd                   gelu: the tanh form
  logits       = t tanh(E N_f(x) / t)
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence, Tuple

import torch

F64 = torch.float64


# ----------------------------------------------------------------------------- small pieces
def rms_norm(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """v over its root mean square along the last dimension, times w."""
    v = v.to(F64)
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps) * w.to(F64)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1.0 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def linear(w: torch.Tensor, h: torch.Tensor, b: Optional[torch.Tensor] = None) -> torch.Tensor:
    """W stored [out, in], applied to every row of h, a bias added."""
    y = h.to(F64) @ w.to(F64).T
    return y if b is None else y + b.to(F64)


# ----------------------------------------------------------------------------- rotation
def stretched(base: float, dims: int, scaling: Optional[dict]) -> Tuple[List[float], float]:
    """The pairs' frequencies and the factor on cosine and sine.  ``scaling``: pairs that turn
    often within the original range keep their frequency, slow ones are slowed by the factor, a
    ramp over the pair's number between."""
    freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freqs, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def number(turns: float) -> float:
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(number(float(scaling["fast"]))), 0)
    hi = min(math.ceil(number(float(scaling["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(z: torch.Tensor, positions: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """z [T, heads, d]: the pairs (i, i + dims/2) of the first ``dims`` elements turned."""
    out = z.to(F64).clone()
    if not rot or not rot["dims"]:
        return out
    half = int(rot["dims"]) // 2
    freqs, length = stretched(float(rot["base"]), int(rot["dims"]), rot.get("scaling"))
    for i in range(half):
        a = positions.to(F64) * freqs[i]
        c, s = length * torch.cos(a)[:, None], length * torch.sin(a)[:, None]
        u, v = z[:, :, i].to(F64), z[:, :, i + half].to(F64)
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- attention
def seen(T: int, size: Optional[int] = None) -> torch.Tensor:
    """[T, T] bool: whether position i sees position j."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    return ok if size is None else ok & (i - j < size)


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float,
           visible: torch.Tensor) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H dv]; H / G neighbouring query heads share
    a key head."""
    T, H, _ = q.shape
    k = k.repeat_interleave(H // k.shape[1], dim=1)
    v = v.repeat_interleave(H // v.shape[1], dim=1)
    s = torch.matmul(q.permute(1, 0, 2), k.permute(1, 2, 0)) * float(scale)
    s = s.masked_fill(~visible, -math.inf)
    a = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    a = a / a.sum(dim=-1, keepdim=True)
    return torch.matmul(a, v.permute(1, 0, 2)).permute(1, 0, 2).reshape(T, -1)


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    H, G, d, dv = (int(m[n]) for n in ("heads", "kv_heads", "dim", "vdim"))
    T = h.shape[0]
    p = torch.arange(T)
    q = rotate(rms_norm(linear(w["q"], h).view(T, H, d), w["q.norm"], eps), p, m.get("rot"))
    k = rotate(rms_norm(linear(w["k"], h).view(T, G, d), w["k.norm"], eps), p, m.get("rot"))
    v = linear(w["v"], h).view(T, G, dv)
    return linear(w["o"], attend(q, k, v, m["scale"], seen(T)))


def latent_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    H, d, dv = (int(m[n]) for n in ("heads", "dim", "vdim"))
    T = h.shape[0]
    q = linear(w["q"], h).view(T, H, d)
    c = rms_norm(linear(w["dkv"], h), w["dkv.norm"], eps)
    k, v = linear(w["uk"], c).view(T, H, d), linear(w["uv"], c).view(T, H, dv)
    size = (m.get("mask") or {}).get("size")
    return linear(w["o"], attend(q, k, v, m["scale"], seen(T, size)))


# ----------------------------------------------------------------------------- the recurrence
def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, C], taps [C, n]: channel by channel over time, zeros before the start; the last tap
    meets the token's own row."""
    T, C = x.shape
    n = taps.shape[1]
    padded = torch.cat([torch.zeros((n - 1, C), dtype=F64), x.to(F64)])
    y = torch.zeros((T, C), dtype=F64)
    for j in range(n):
        y = y + padded[j:j + T] * taps[:, j].to(F64)
    return y + bias.to(F64)


def state_space(x, B, C, dt, A_log, D, state=None):
    """x [T, H, dv], B and C [T, G, N], dt [T, H] (behind its softplus), A_log and D [H].  Returns
    (y [T, H, dv], S [H, N, dv])."""
    T, H, dv = x.shape
    x, dt = x.to(F64), dt.to(F64)
    B = B.to(F64).repeat_interleave(H // B.shape[1], dim=1)
    C = C.to(F64).repeat_interleave(H // C.shape[1], dim=1)
    rate = torch.exp(A_log.to(F64))
    S = torch.zeros((H, B.shape[2], dv), dtype=F64) if state is None else state.to(F64).clone()
    y = torch.zeros((T, H, dv), dtype=F64)
    for t in range(T):
        decay = torch.exp(-rate * dt[t])[:, None, None]
        S = decay * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t][:, :, None]).sum(dim=1) + D.to(F64)[:, None] * x[t]
    return y, S


def gated_parts_norm(y, z, w, parts: int, eps: float) -> torch.Tensor:
    """y silu(z), every one of ``parts`` equal parts of a row over its own root mean square, times
    w [row]."""
    u = (y.to(F64) * silu(z.to(F64)))
    T, W = u.shape
    u = rms_norm(u.view(T, parts, W // parts), torch.ones(W // parts, dtype=F64), eps)
    return u.reshape(T, W) * w.to(F64)


def mamba2_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    H, dv, N, G = (int(m[n]) for n in ("heads", "vdim", "state", "groups"))
    T, inner = h.shape[0], H * dv
    z, xbc, s = torch.split(linear(w["in"], h), [inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=1)
    y, _ = state_space(x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N),
                       softplus(s + w["dt_bias"].to(F64)), w["A_log"], w["D"])
    return linear(w["o"], gated_parts_norm(y.reshape(T, inner), z, w["norm"],
                                           int(m["norm_groups"]), eps))


# ----------------------------------------------------------------------------- the model
def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return linear(w["down"], gelu_tanh(linear(w["gate"], h, w["gate.b"]))
                  * linear(w["up"], h, w["up.b"]), w["down.b"])


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer, "mamba2": mamba2_mixer}


def below(tensors: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {n[len(prefix):]: t for n, t in tensors.items() if n.startswith(prefix)}


def owner(config: dict, i: int) -> int:
    """The layer whose tensors layer i runs with."""
    while config["layers"][i].get("weights_of") is not None:
        i = int(config["layers"][i]["weights_of"])
    return i


def layer(i: int, x: torch.Tensor, config: dict, tensors) -> torch.Tensor:
    L, eps = config["layers"][i], float(config["norm"]["eps"])
    w = below(tensors, f"l{owner(config, i)}.")
    y = MIXERS[L["type"]](rms_norm(x, w["norm1"], eps), below(w, "mix."), L["mixer"], eps)
    x = x + rms_norm(y, w["norm1b"], eps)
    if L.get("mlp") is not None:
        y = feed_forward(rms_norm(x, w["norm2"], eps), below(w, "mlp."))
        x = x + rms_norm(y, w["norm2b"], eps)
    return x


def embedding(token_ids: Sequence[int], config: dict, tensors) -> torch.Tensor:
    ids = torch.tensor(list(token_ids), dtype=torch.long)
    return rms_norm(tensors["embed"].to(F64)[ids], tensors["embed.norm"],
                    float(config["norm"]["eps"]))


def forward(token_ids: Sequence[int], config: dict, tensors,
            after_layers: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; ``after_layers`` takes the stream after every
    layer."""
    x = embedding(token_ids, config, tensors)
    for i in range(len(config["layers"])):
        x = layer(i, x, config, tensors)
        if after_layers is not None:
            after_layers.append(x.clone())
    x = rms_norm(x, tensors["final.norm"], float(config["norm"]["eps"]))
    logits = linear(tensors["embed"], x)
    cap = config.get("logit_softcap")
    return logits if cap is None else float(cap) * torch.tanh(logits / float(cap))


def greedy(prompt: Sequence[int], n: int, config: dict, tensors) -> List[int]:
    out = list(prompt)
    for _ in range(n):
        out.append(int(torch.argmax(forward(out, config, tensors)[-1])))
    return out[len(prompt):]
