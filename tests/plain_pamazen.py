"""The Pamazen decoder, plainly: whole sequences, no cache, float64, one function per mechanism.

It shares nothing with the package: a model is a configuration (the dict that config.json holds) and a dict of
tensors by their names in a file.  ``round_to=torch.bfloat16`` rounds what a bfloat16 engine stores between its
kernels, which tells how far rounding alone moves the logits.

Notation.  W: the stream's width; X [S, T, W] the S streams, all equal to the embedding's rows at the start; m the
residual multiplier.  A sublayer f with the vectors a, b [S] and the matrix M [from, to]:

    u = sum_s a_s X_s,      y = f(g n(u)),      X_t <- sum_s M[s, t] X_s + m b_t y,

n(y) = y / sqrt(mean(y^2) + eps), g one number.  At the end x = sum_s X_s.
"""
from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional, Tuple

import torch

F64 = torch.float64


def _r(x: torch.Tensor, round_to) -> torch.Tensor:
    return x if round_to is None else x.to(round_to).to(F64)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def softcap(x: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(x / cap)


# ---------------------------------------------------------------------------------------------- attention
def rotation_angles(positions: torch.Tensor, dims: int, base: float, factor: float = 1.0) -> torch.Tensor:
    """[T, dims / 2]: position times base^(-2i/dims) / factor."""
    i = torch.arange(dims // 2, dtype=F64)
    return positions.to(F64)[:, None] * (base ** (-2.0 * i / dims) / factor)[None, :]


def rotate_pairs(x: torch.Tensor, angles: torch.Tensor, dims: int) -> torch.Tensor:
    """x [T, heads, d]: value 2i and value 2i + 1 of the first ``dims`` values of every head turn by angle i."""
    out = x.clone()
    cos, sin = torch.cos(angles)[:, None, :], torch.sin(angles)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def seen_keys(T: int, size: Optional[int] = None, keep_first: int = 0) -> torch.Tensor:
    """[T, T] bool (query i, key j): j <= i, and with a window j within the last ``size`` or among the first
    ``keep_first``."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    seen = j <= i
    if size is not None:
        seen = seen & ((i - j < size) | (j < keep_first))
    return seen


def sink_softmax(scores: torch.Tensor, seen: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Softmax over the seen keys whose denominator also holds exp(sink)."""
    s = scores.masked_fill(~seen, -math.inf)
    top = torch.maximum(s.max(dim=1, keepdim=True).values, sink)
    ex = torch.exp(s - top)
    return ex / (ex.sum(dim=1, keepdim=True) + torch.exp(sink - top))


def grouped_attention(q, k, v, scale, seen, sinks, cap=None) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H dv]; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale
        if cap is not None:
            s = softcap(s, cap)
        out[:, h] = sink_softmax(s, seen, sinks[h]) @ v[:, g]
    return out.reshape(T, -1)


def attention_mixer(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, shared: dict,
                    round_to=None) -> torch.Tensor:
    """Rotated pairs, one more in the softmax's denominator, values mixed with those of the first layer that mixes
    (which leaves them in ``shared``)."""
    T = a.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = _r(a @ w[p + "q"].T, round_to).view(T, H, d)
    k = _r(a @ w[p + "k"].T, round_to).view(T, G, d)
    v = _r(a @ w[p + "v"].T, round_to)
    rot = m.get("rot")
    if rot and rot["dims"]:
        ang = rotation_angles(torch.arange(T), rot["dims"], float(rot["base"]), float((rot.get("scaling") or {}).get("factor", 1.0)))
        q, k = _r(rotate_pairs(q, ang, rot["dims"]), round_to), _r(rotate_pairs(k, ang, rot["dims"]), round_to)
    if m.get("v_mix"):
        if "v_first" in shared:
            lam = w[p + "vmix"]
            v = _r((1.0 - lam) * v + lam * shared["v_first"], round_to)
        else:
            shared["v_first"] = v
    o = grouped_attention(q, k, v.view(T, G, dv), m["scale"], seen_keys(T), torch.zeros(H, dtype=F64))
    return _r(o, round_to) @ w[p + "o"].T


def window_attention(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, round_to=None,
                     scale: float = 1.0) -> torch.Tensor:
    """Values are the projected keys; a norm per query and key head; capped scores; a window with kept first
    positions; a learned sink.  ``scale`` multiplies the result."""
    T = a.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q = _r(a @ w[p + "q"].T, round_to).view(T, H, d)
    k = _r(a @ w[p + "k"].T, round_to).view(T, G, d)
    v = _r(k * scale, round_to)
    q = _r(unit_rms(q, eps) * w[p + "q.norm"], round_to)
    k = _r(unit_rms(k, eps) * w[p + "k.norm"], round_to)
    mask = m.get("mask")
    seen = seen_keys(T, int(mask["size"]), int(mask["keep_first"])) if mask else seen_keys(T)
    o = grouped_attention(q, k, v, m["scale"], seen, w[p + "sink"], float(m["softcap"]) if m.get("softcap") else None)
    return _r(o, round_to) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- the recurrence
def unit_keys(k: torch.Tensor) -> torch.Tensor:
    return k / torch.sqrt((k * k).sum(dim=-1, keepdim=True) + 1e-6)


def delta_recurrence(r, k, v, w, a, state: Optional[torch.Tensor] = None):
    """One head, token after token: S <- diag(w_t) S - (a_t * u_t) (u_t^T S) + k_t v_t^T with both terms reading the
    old S, o_t = S^T r_t; r, k, w, a [T, d], v [T, dv], u_t the unit key."""
    T, d = r.shape
    S = torch.zeros((d, v.shape[1]), dtype=F64) if state is None else state.clone()
    u = unit_keys(k)
    out = torch.empty((T, v.shape[1]), dtype=F64)
    for t in range(T):
        S = w[t][:, None] * S - (a[t] * u[t])[:, None] * (u[t] @ S)[None, :] + k[t][:, None] * v[t][None, :]
        out[t] = S.T @ r[t]
    return out, S


def delta_decays(x: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, round_to=None) -> torch.Tensor:
    mid = _r(torch.tanh(_r(x @ w[p + "w1"].T, round_to)), round_to)
    return torch.exp(-math.exp(-0.5) * sigmoid(mid @ w[p + "w2"].T + w[p + "w0"]))


def delta_mixer(x: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, round_to=None,
                scale: float = 1.0) -> torch.Tensor:
    T, H, d = x.shape[0], m["heads"], m["dim"]
    r, k, v, g, za = (_r(x @ w[p + n].T, round_to) for n in ("r", "k", "v", "g", "a"))
    decay = delta_decays(x, w, p, round_to).view(T, H, d)
    a = sigmoid(za + w[p + "a.b"]).view(T, H, d)
    r, k, v = r.view(T, H, d), k.view(T, H, d), v.view(T, H, d)
    out = torch.empty((T, H, d), dtype=F64)
    for h in range(H):
        o, _ = delta_recurrence(r[:, h], k[:, h], v[:, h], decay[:, h], a[:, h])
        out[:, h] = unit_rms(o, eps)
    y = out.reshape(T, H * d) * w[p + "norm"] * sigmoid(g) * scale
    return _r(y, round_to) @ w[p + "o"].T


def parallel_mixer(a: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, eps: float, shared: dict,
                   round_to=None) -> torch.Tensor:
    return (window_attention(a, w, p + "left.", m["left"], eps, round_to, float(m["left_scale"]))
            + delta_mixer(a, w, p + "right.", m["right"], eps, round_to, float(m["right_scale"])))


MIXERS = {"attention": attention_mixer, "parallel": parallel_mixer}


# ---------------------------------------------------------------------------------------------- experts
def choose_experts(s: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int):
    """s [T, E] the softmax over all experts.  Returns (ids, weights) [T, top] by falling choice score."""
    T, E = s.shape
    choice = s + correction
    size = E // groups
    best = choice.view(T, groups, size).max(dim=2).values
    kept = torch.zeros((T, groups), dtype=torch.bool)
    kept.scatter_(1, best.topk(keep, dim=1).indices, True)
    masked = choice.masked_fill(~kept.repeat_interleave(size, dim=1), -math.inf)
    ids = masked.topk(top, dim=1).indices
    return ids, s.gather(1, ids)


def gated_expert(f: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, round_to=None) -> torch.Tensor:
    return _r(silu(f @ w[p + "gate"].T) * (f @ w[p + "up"].T), round_to) @ w[p + "down"].T


def routed_experts(f: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, m: Mapping, round_to=None,
                   margins: Optional[list] = None) -> torch.Tensor:
    r = m["router"]
    E, top = r["experts"], r["top"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.softmax(f @ w[p + "router"].T, dim=1)
    ids, wts = choose_experts(s, w[p + "correction"], top, groups["count"], groups["keep"])
    if margins is not None:
        margins.append(choice_margin(s, w[p + "correction"], top, groups["count"], groups["keep"]))
    out = torch.zeros_like(f)
    for e in range(E + int(r.get("identity") or 0)):
        wt = (wts * (ids == e)).sum(dim=1)
        took = (ids == e).any(dim=1)
        if took.any():
            y = f[took] if e >= E else gated_expert(f[took], w, f"{p}e{e}.", round_to)
            out[took] += wt[took, None] * y
    if m.get("shared"):
        out = out + sigmoid(f @ w[p + "shared.sg"].T) * gated_expert(f, w, p + "shared.", round_to)
    return out


def choice_margin(s: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int) -> torch.Tensor:
    """[T]: by how much the choice of experts (or of groups) would have to move to come out differently."""
    T, E = s.shape
    choice = s + correction
    size = E // groups
    best = choice.view(T, groups, size).max(dim=2).values
    out = torch.full((T,), math.inf, dtype=F64)
    if keep < groups:
        o = best.sort(dim=1, descending=True).values
        out = torch.minimum(out, o[:, keep - 1] - o[:, keep])
    kept = torch.zeros((T, groups), dtype=torch.bool)
    kept.scatter_(1, best.topk(keep, dim=1).indices, True)
    o = choice.masked_fill(~kept.repeat_interleave(size, dim=1), -math.inf).sort(dim=1, descending=True).values
    if top < E:
        out = torch.minimum(out, o[:, top - 1] - o[:, top])
    return out


# ---------------------------------------------------------------------------------------------- streams and the model
def hyper_read(X: torch.Tensor, a: torch.Tensor) -> torch.Tensor:
    return torch.einsum("s,stw->tw", a, X)


def hyper_write(X: torch.Tensor, y: torch.Tensor, mix: torch.Tensor, b: torch.Tensor, mult: float) -> torch.Tensor:
    return torch.einsum("st,snw->tnw", mix, X) + mult * b[:, None, None] * y[None]


def forward(cfg: Mapping, w: Mapping[str, torch.Tensor], tokens, round_to=None, streams: Optional[list] = None,
            upto: Optional[int] = None, margins: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  ``streams``: gets the sum of the streams after every layer.
    ``upto``: only the first so many layers."""
    w = {k: (v.to(F64) if v.dtype.is_floating_point else v) for k, v in w.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    X = w["embed"][tokens][None].repeat(int(cfg["streams"]), 1, 1)
    shared: dict = {}
    for i, layer in enumerate(cfg["layers"]):
        if upto is not None and i >= upto:
            break
        p = f"l{i}."
        f = _r(unit_rms(hyper_read(X, w[p + "hc1.in"]), eps) * w[p + "norm1"], round_to)
        y = MIXERS[layer["type"]](f, w, p + "mix.", layer["mixer"], eps, shared, round_to)
        X = hyper_write(X, y, w[p + "hc1.mix"], w[p + "hc1.out"], mult)
        if layer.get("mlp") is not None:
            f = _r(unit_rms(hyper_read(X, w[p + "hc2.in"]), eps) * w[p + "norm2"], round_to)
            y = routed_experts(f, w, p + "mlp.", layer["mlp"], round_to, margins)
            X = hyper_write(X, y, w[p + "hc2.mix"], w[p + "hc2.out"], mult)
        if streams is not None:
            streams.append(X.sum(dim=0))
    x = X.sum(dim=0)
    z = _r(unit_rms(x, eps) * w["final.norm"], round_to) @ w["head"].T
    cap = cfg.get("logit_softcap")
    return softcap(z, float(cap)) if cap else z


# ---------------------------------------------------------------------------------------------- weights for tests
def tensor_shapes(cfg: Mapping, rank: int = 12) -> Dict[str, Tuple[int, ...]]:
    """Names and shapes of a model's tensors.  ``rank``: the middle of the decays' two products."""
    V, W, S = cfg["vocab"], cfg["width"], cfg["streams"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (V, W)}

    def hyper(p):
        out.update({p + "in": (S,), p + "out": (S,), p + "mix": (S, S)})

    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = ()
        hyper(p + "hc1.")
        if layer["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out.update({p + "mix.q": (H * d, W), p + "mix.k": (G * d, W), p + "mix.v": (G * dv, W), p + "mix.o": (W, H * dv)})
            if m.get("v_mix"):
                out[p + "mix.vmix"] = ()
        else:
            l, H, G, d = p + "mix.left.", m["left"]["heads"], m["left"]["kv_heads"], m["left"]["dim"]
            out.update({l + "q": (H * d, W), l + "k": (G * d, W), l + "q.norm": (d,), l + "k.norm": (d,), l + "sink": (H,),
                        l + "o": (W, H * d)})
            r, n = p + "mix.right.", m["right"]["heads"] * m["right"]["dim"]
            out.update({r + x: (n, W) for x in ("r", "k", "v", "g", "a")})
            out.update({r + "a.b": (n,), r + "w1": (rank, W), r + "w2": (n, rank), r + "w0": (n,), r + "norm": (n,),
                        r + "o": (W, n)})
        f = layer.get("mlp")
        if f is not None:
            out[p + "norm2"] = ()
            hyper(p + "hc2.")
            E = f["router"]["experts"]
            total = E + int(f["router"].get("identity") or 0)
            q = p + "mlp."
            for pre, ff in [(f"e{e}.", f["expert"]["ff"]) for e in range(E)] + ([("shared.", f["shared"]["ff"])] if f.get("shared") else []):
                out.update({q + pre + "gate": (ff, W), q + pre + "up": (ff, W), q + pre + "down": (W, ff)})
            out.update({q + "router": (total, W), q + "correction": (total,)})
            if f.get("shared"):
                out[q + "shared.sg"] = (1, W)
    out["final.norm"] = ()
    out["head"] = (V, W)
    return out


def random_weights(cfg: Mapping, seed: int = 0, store: torch.dtype = torch.bfloat16, rank: int = 12) -> Dict[str, torch.Tensor]:
    """Weights of a size that keeps every branch of order one; rounded to ``store``."""
    g = torch.Generator().manual_seed(seed)
    S = cfg["streams"]
    out = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        last = name.rsplit(".", 1)[-1]
        rnd = lambda: torch.randn(shape, generator=g)                               # noqa: E731
        if "norm" in last:
            t = 1.0 + 0.2 * rnd()
        elif ".hc" in name:
            if last == "mix":
                t = torch.eye(S) + 0.15 * rnd()
            else:
                t = (1.0 / S if last == "in" else 1.0) * (1.0 + 0.4 * rnd())
        elif last == "w0":
            t = -4.0 + 5.0 * torch.rand(shape, generator=g)         # decays between slow and fast
        elif last == "b":
            t = rnd()
        elif last == "correction":
            t = 0.1 * rnd()
        elif last == "sink":
            t = rnd()
        elif last == "vmix":
            t = 0.2 + 0.6 * torch.rand(shape, generator=g)
        elif name == "embed":
            t = rnd()
        elif last == "router":
            t = 2.0 * rnd() / math.sqrt(shape[-1])
        elif last in ("q", "k") and ".right." not in name:
            t = 1.5 * rnd() / math.sqrt(shape[-1])                  # scores of some size, so that the masks matter
        elif last == "k":
            t = 0.5 * rnd() / math.sqrt(shape[-1])                  # what a token writes, of the size of what it removes
        else:
            t = rnd() / math.sqrt(shape[-1])
        out[name] = t.to(store)
    return out
