"""The Mirovik decoder, plainly: whole sequences, no cache, float64, one function per mechanism.

It shares nothing with the package: a model is a configuration (the dict that config.json holds) and a dict of
tensors by their names in a file.  ``round_to=torch.bfloat16`` rounds what a bfloat16 engine stores between its
kernels, which tells how far rounding alone moves the logits.

Notation.  n(y, w) = y / sqrt(mean(y^2) + eps) * (1 + w).  A layer with the mixer M and the feed-forward F:

    x <- x + n(M(n(x, w1)), w1b),        x <- x + n(F(n(x, w2)), w2b).

A stretch of layers runs several times; before its pass t the vector r_t is added to x.
"""
from __future__ import annotations

import math
from fractions import Fraction
from typing import Dict, List, Mapping, Optional, Tuple

import torch

F64 = torch.float64


def _r(x: torch.Tensor, round_to) -> torch.Tensor:
    return x if round_to is None else x.to(round_to).to(F64)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def offset_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def gelu_tanh(x: torch.Tensor) -> torch.Tensor:
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


# ---------------------------------------------------------------------------------------------- attention
def bucket_of(n: int, buckets: int, far) -> int:
    """The row of the bias table for a key n places back: the first half of the rows one each, the others in steps
    that grow geometrically up to the distance ``far``.  Worked out with whole numbers: the largest k <= B - h with
    (n / h)^(B - h) >= (far / h)^k, h = B / 2."""
    h = buckets // 2
    if n < h:
        return n
    far = Fraction(far)
    left, k = Fraction(n, h) ** (buckets - h), 0
    while k < buckets - h and left >= (far / h) ** (k + 1):
        k += 1
    return min(buckets - 1, h + k)


def distance_bias(T: int, rel: torch.Tensor, far) -> torch.Tensor:
    """[heads, T, T]: (h, i, j) -> rel[bucket(i - j), h]; zero above the diagonal."""
    rows = torch.tensor([bucket_of(n, rel.shape[0], far) for n in range(T)])
    d = (torch.arange(T)[:, None] - torch.arange(T)[None, :])
    return torch.where((d >= 0)[None], rel[rows[d.clamp(min=0)]].permute(2, 0, 1), torch.zeros((), dtype=F64))


def biased_attention(q, k, v, scale: float, bias: torch.Tensor) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv], bias [H, T, T] -> [T, H dv]; query head h reads head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    seen = torch.ones((T, T), dtype=torch.bool).tril()
    out = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale + bias[h]
        out[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), dim=1) @ v[:, g]
    return out.reshape(T, -1)


def attention_mixer(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, round_to=None,
                    scale: float = 1.0) -> torch.Tensor:
    """Queries and keys normed over all heads at once, a distance bias, a gate per value; ``scale`` multiplies the
    result."""
    T = a.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v, g = (_r(a @ w[p + n].T, round_to) for n in ("q", "k", "v", "g"))
    q = _r(unit_rms(q, eps) * w[p + "q.norm"], round_to).view(T, H, d)
    k = _r(unit_rms(k, eps) * w[p + "k.norm"], round_to).view(T, G, d)
    o = biased_attention(q, k, v.view(T, G, dv), float(m["scale"]), distance_bias(T, w[p + "rel"], m["bias_max"]))
    return _r(o * sigmoid(g) * scale, round_to) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- retention
def rotate_half(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, d]: values i and i + dims / 2 of every head turn by position * base^(-2i / dims)."""
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=F64) / max(dims, 1))
    a = (positions.to(F64)[:, None] * f[None, :])[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., dims:]], dim=-1)


def retention(q, k, v, decay: float, state: Optional[torch.Tensor] = None):
    """One head, token after token: S <- decay S + k_t v_t^T, o_t = S^T q_t."""
    T, d = q.shape
    S = torch.zeros((d, v.shape[1]), dtype=F64) if state is None else state.clone()
    out = torch.empty((T, v.shape[1]), dtype=F64)
    for t in range(T):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out[t] = S.T @ q[t]
    return out, S


def retention_mixer(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, round_to=None,
                    scale: float = 1.0) -> torch.Tensor:
    T, H, d, dv = a.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v, g = (_r(a @ w[p + n].T, round_to) for n in ("q", "k", "v", "g"))
    q, k, v = q.view(T, H, d), k.view(T, H, d), v.view(T, H, dv)
    rot = m.get("rot")
    if rot and rot["dims"]:
        pos = torch.arange(T)
        q = rotate_half(q, pos, rot["dims"], float(rot["base"]))
        k = rotate_half(k, pos, rot["dims"], float(rot["base"]))
    k = k * d ** -0.5
    o = torch.stack([unit_rms(retention(q[:, h], k[:, h], v[:, h], float(m["decay"][h]))[0], eps) for h in range(H)], dim=1)
    return _r(o.reshape(T, -1) * silu(g) * scale, round_to) @ w[p + "o"].T


def parallel_mixer(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, round_to=None) -> torch.Tensor:
    return (attention_mixer(a, w, p + "left.", m["left"], eps, round_to, float(m["left_scale"]))
            + retention_mixer(a, w, p + "right.", m["right"], eps, round_to, float(m["right_scale"])))


# ---------------------------------------------------------------------------------------------- the selective scan
def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, C], taps [C, K], the last column for the token itself, zeros before the start."""
    T, K = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros((K - 1, x.shape[1]), dtype=F64), x], dim=0)
    return sum(padded[j:j + T] * taps[:, j] for j in range(K)) + bias


def selective_scan(x, dt, A, B, C, D, state: Optional[torch.Tensor] = None):
    """x, dt [T, C], A [C, n], B, C [T, n]: S <- exp(dt A) S + dt x B, y = S C + D x, token after token."""
    S = torch.zeros(A.shape, dtype=F64) if state is None else state.clone()
    y = torch.empty_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba_mixer(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, round_to=None) -> torch.Tensor:
    I, R, n = m["inner"], m["dt_rank"], m["state"]
    xz = _r(a @ w[p + "in"].T, round_to)
    x, z = xz[:, :I], xz[:, I:]
    x = _r(silu(causal_conv(x, w[p + "conv"], w[p + "conv.b"])), round_to)
    low = _r(x @ w[p + "x"].T, round_to)
    dt = softplus(low[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(w[p + "A_log"]), low[:, R:R + n], low[:, R + n:], w[p + "D"])
    return _r(y * silu(z), round_to) @ w[p + "o"].T


MIXERS = {"parallel": parallel_mixer, "mamba1": mamba_mixer}


# ---------------------------------------------------------------------------------------------- feed-forward
def dense_mlp(f: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, round_to=None) -> torch.Tensor:
    return _r(gelu_tanh(f @ w[p + "up"].T), round_to) @ w[p + "down"].T


def gated_expert(f: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, round_to=None) -> torch.Tensor:
    return _r(silu(f @ w[p + "gate"].T) * (f @ w[p + "up"].T), round_to) @ w[p + "down"].T


def routed_experts(f: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, round_to=None,
                   margins: Optional[list] = None) -> torch.Tensor:
    """Sigmoid scores, the largest chosen, their scores as they are on the experts' INPUTS; a shared expert."""
    E, top = m["router"]["experts"], m["router"]["top"]
    s = sigmoid(f @ w[p + "router"].T)
    wts, ids = s.topk(top, dim=1)
    if margins is not None:
        o = s.sort(dim=1, descending=True).values
        margins.append(o[:, top - 1] - o[:, top] if top < E else torch.full((f.shape[0],), math.inf, dtype=F64))
    out = torch.zeros_like(f)
    for e in range(E):
        took = (ids == e).any(dim=1)
        if took.any():
            wt = (wts * (ids == e)).sum(dim=1)[took]
            out[took] += gated_expert(wt[:, None] * f[took], w, f"{p}e{e}.", round_to)
    if m.get("shared"):
        out = out + gated_expert(f, w, p + "shared.", round_to)
    return out


# ---------------------------------------------------------------------------------------------- the model
def layer_runs(cfg: Mapping) -> List[Tuple[int, Optional[int]]]:
    """(layer, the pass of the loop that begins with this run, or None), in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(cfg: Mapping, w: Mapping[str, torch.Tensor], tokens, round_to=None, streams: Optional[list] = None,
            upto: Optional[int] = None, margins: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  ``streams``: gets the stream after every layer run.  ``upto``: only
    the first so many layer runs."""
    w = {k: (v.to(F64) if v.dtype.is_floating_point else v) for k, v in w.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][tokens] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    for run, (i, t) in enumerate(layer_runs(cfg)):
        if upto is not None and run >= upto:
            break
        layer, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = x + w["loop.step"][t]
        f = _r(offset_norm(x, w[p + "norm1"], eps), round_to)
        x = x + offset_norm(_r(MIXERS[layer["type"]](f, w, p + "mix.", layer["mixer"], eps, round_to), round_to),
                            w[p + "norm1b"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            f = _r(offset_norm(x, w[p + "norm2"], eps), round_to)
            y = routed_experts(f, w, p + "mlp.", mlp, round_to, margins) if mlp["kind"] == "moe" else \
                dense_mlp(f, w, p + "mlp.", round_to)
            x = x + offset_norm(_r(y, round_to), w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x)
    return _r(offset_norm(x, w["final.norm"], eps), round_to) @ w["embed"].T


# ---------------------------------------------------------------------------------------------- weights for tests
def tensor_shapes(cfg: Mapping, buckets: int = 20) -> Dict[str, Tuple[int, ...]]:
    """Names and shapes of a model's tensors.  ``buckets``: rows of the bias tables."""
    V, W = cfg["vocab"], cfg["width"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (V, W)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], W)
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        out.update({p + n: (W,) for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ())})
        if layer["type"] == "mamba1":
            I, R, n, q = m["inner"], m["dt_rank"], m["state"], p + "mix."
            out.update({q + "in": (2 * I, W), q + "conv": (I, m["conv"]), q + "conv.b": (I,), q + "x": (R + 2 * n, I),
                        q + "dt": (I, R), q + "dt.b": (I,), q + "A_log": (I, n), q + "D": (I,), q + "o": (W, I)})
        else:
            l, q = m["left"], p + "mix.left."
            H, G, d, dv = l["heads"], l["kv_heads"], l["dim"], l["vdim"]
            out.update({q + "q": (H * d, W), q + "k": (G * d, W), q + "v": (G * dv, W), q + "q.norm": (H * d,),
                        q + "k.norm": (G * d,), q + "rel": (int(l.get("buckets", buckets)), H), q + "g": (H * dv, W),
                        q + "o": (W, H * dv)})
            r, q = m["right"], p + "mix.right."
            H, d, dv = r["heads"], r["dim"], r["vdim"]
            out.update({q + "q": (H * d, W), q + "k": (H * d, W), q + "v": (H * dv, W), q + "g": (H * dv, W), q + "o": (W, H * dv)})
        if f is not None:
            q = p + "mlp."
            if f["kind"] == "dense":
                out.update({q + "up": (f["ff"], W), q + "down": (W, f["ff"])})
            else:
                E = f["router"]["experts"]
                for pre, ff in [(f"e{e}.", f["expert"]["ff"]) for e in range(E)] + ([("shared.", f["shared"]["ff"])] if f.get("shared") else []):
                    out.update({q + pre + "gate": (ff, W), q + pre + "up": (ff, W), q + pre + "down": (W, ff)})
                out[q + "router"] = (E, W)
    out["final.norm"] = (W,)
    return out


def random_weights(cfg: Mapping, seed: int = 0, store: torch.dtype = torch.bfloat16, buckets: int = 20) -> Dict[str, torch.Tensor]:
    """Weights of a size that keeps every branch of order one; rounded to ``store``."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, buckets).items():
        last = name.rsplit(".", 1)[-1]
        rnd = lambda: torch.randn(shape, generator=g)                               # noqa: E731
        uni = lambda: torch.rand(shape, generator=g)                                # noqa: E731
        if name.endswith((".q.norm", ".k.norm")):
            t = 1.0 + 0.2 * rnd()
        elif "norm" in last:
            t = 0.2 * rnd()
        elif last == "rel":
            t = 1.5 * rnd()
        elif name == "loop.step":
            t = 0.5 * rnd()
        elif last == "A_log":
            t = torch.log(torch.arange(1, shape[1] + 1, dtype=torch.float32))[None, :] + 0.3 * rnd()
        elif name.endswith("dt.b"):
            t = -4.0 + 4.0 * uni()                  # steps between slow and fast
        elif last == "b":
            t = 0.3 * rnd()
        elif last == "D":
            t = 0.5 + uni()
        elif last == "conv":
            t = rnd() / math.sqrt(shape[-1])
        elif name == "embed":
            t = rnd() / math.sqrt(shape[-1])
        elif last == "router":
            t = 2.0 * rnd() / math.sqrt(shape[-1])
        elif name.endswith(".right.k"):
            # a token's own key lies along its query: what a retention head reads is then no difference of nearly equal
            # terms, which the division by its root mean square would blow up
            t = 0.7 * out[name[:-1] + "q"].float() + 0.7 * rnd() / math.sqrt(shape[-1])
        else:
            t = rnd() / math.sqrt(shape[-1])
        out[name] = t.to(store)
    return out
