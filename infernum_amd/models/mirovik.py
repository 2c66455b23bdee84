"""The Mirovik decoder as a ModelSpec: layers with a norm before and after each sublayer (``sandwich``), norms whose stored
weight lies around zero; the mixer is attention beside retention on the same input (``side_by_side``: ``softmax_attention``
with queries and keys normed over all heads, a learned bias by distance and a gate per value, and ``retention``), or a
selective scan (``mamba1``); the feed-forward is dense (the tanh form of GELU), routed experts behind a sigmoid router whose
weights stand on the experts' inputs, with a shared expert, or absent; a stretch of layers may run several times with the
same tensors, every pass with a cache and state of its own and a learned vector added to the stream before it; the head is
the embedding table.  Tensor names: ``embed``, ``loop.step``, ``final.norm``, ``l<i>.norm1|norm1b|norm2|norm2b``,
``l<i>.mix.*`` (``l<i>.mix.left.*|right.*``), ``l<i>.mlp.*``.
"""
from __future__ import annotations

from ..config.mirovik import MIROVIK_MODEL_TYPE, MirovikConfig, ParallelConfig
from ..config.registry import register_architecture
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

DENSE_ACTIVATION = "gelu_tanh"          # fixed by the design


def _rope(base: float, dims: int, head_dim: int) -> dict:
    if dims == 0:
        return {"kind": "none"}
    return {"kind": "rope", "params": {"head_dim": head_dim, "theta": base, "rotary_dim": dims, "pairing": "half"}}


def mirovik_model_spec(cfg: MirovikConfig, init_std: float = 0.05) -> ModelSpec:
    W = cfg.width

    def norm(prefix: str) -> PartSpec:
        return PartSpec("rmsnorm", {"size": W, "eps": cfg.norm_eps, "init": ("uniform", -0.2, 0.2), "name": "",
                                    "unit_offset": True}, prefix)

    layers, ignored = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        if isinstance(m, ParallelConfig):
            left, right = m.left, m.right
            mixer = PartSpec("side_by_side", {"hidden_size": W, "mixers": {
                "left": {"kind": "softmax_attention", "scale": m.left_scale, "params": {
                    "hidden_size": W, "num_heads": left.heads, "num_kv_heads": left.kv_heads, "head_dim": left.dim,
                    "value_dim": left.vdim, "scale": left.scale, "qk_norm": "rows", "norm_eps": cfg.norm_eps,
                    "distance_bias": {"far": left.bias_max, "rows": left.buckets, "name": "rel"}, "output_gate": True,
                    "init_std": init_std}},
                "right": {"kind": "retention", "scale": m.right_scale, "params": {
                    "hidden_size": W, "num_heads": right.heads, "head_dim": right.dim, "value_dim": right.vdim,
                    "decay": right.decay, "norm_eps": cfg.norm_eps,
                    "position": _rope(right.rot_base, right.rot_dims, right.dim), "init_std": init_std}}}}, p + "mix.")
        else:
            mixer = PartSpec("mamba1", {"hidden_size": W, "inner": m.inner, "state_size": m.state, "dt_rank": m.dt_rank,
                                        "conv_taps": m.conv, "init_std": init_std}, p + "mix.")
        ff, f = None, layer.mlp
        if f is not None and f.kind == "dense":
            ff = PartSpec("dense", {"hidden_size": W, "intermediate_size": f.ff, "activation": DENSE_ACTIVATION,
                                    "names": ("up", "down"), "init_std": init_std}, p + "mlp.")
        elif f is not None:
            ff = PartSpec("routed_experts", {
                "hidden_size": W, "intermediate_size": f.ff, "num_experts": f.experts, "top": f.top, "gated": True,
                "limit": None, "alpha": 1.0, "up_shift": 0.0, "router": "softmax_top", "scores": "sigmoid", "renorm": False,
                "correction_name": None, "weights_on": "input", "shared_ff": f.shared_ff, "init_std": init_std}, p + "mlp.")
        extra = {"mixer_post_norm": norm(p + "norm1b")}
        if ff is not None:
            extra["feed_forward_post_norm"] = norm(p + "norm2b")
        else:                               # no use for the second pair of norms, whether the file has them or not
            ignored += [p + "norm2", p + "norm2b"]
        if cfg.loop is not None and cfg.loop.stop > cfg.loop.start and i == cfg.loop.start:
            extra["stream_in"] = ("stream_in", PartSpec("pass_vector", {"hidden_size": W, "passes": cfg.loop.times,
                                                                        "name": "step", "init_std": 0.3}, "loop."))
        layers.append(LayerSpec(block="sandwich", mixer=mixer, feed_forward=ff, mixer_norm=norm(p + "norm1"),
                                feed_forward_norm=norm(p + "norm2") if ff is not None else None, extra=extra))
    if cfg.loop is not None and cfg.loop.stop <= cfg.loop.start:
        ignored.append("loop.step")
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=W,
        embedding=PartSpec("token", {"vocab_size": cfg.vocab, "hidden_size": W, "scale": cfg.embedding_scale, "name": "",
                                     "init_std": W ** -0.5}, "embed"),
        layers=layers, schedule=[ScheduleEntry(i, pass_index=t) for i, t in cfg.layer_runs()],
        final_norm=norm("final.norm"),
        # the table itself, without its scale
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "", "fallback": "embed", "tied": True,
                                 "init_std": W ** -0.5}, "head"),
        ignored_tensors=tuple(ignored),
    )


register_architecture(MIROVIK_MODEL_TYPE, MirovikConfig, mirovik_model_spec)
