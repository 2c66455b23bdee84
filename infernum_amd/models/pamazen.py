"""The Pamazen decoder as a ModelSpec: several copies of the residual stream that every sublayer reads a mixture of and
writes to (``hyper``), norms with a single number as their weight; the mixer is two mixers side by side on the same input
(``side_by_side``: window attention with kept first positions, a sink, capped scores and the keys as values, and the
generalized delta rule), or attention with rotated pairs, one more in its denominator and values mixed with an earlier
layer's (``softmax_attention``); routed experts behind a softmax router with groups, a correction that moves the choice
only, identity experts and a gated shared expert, or no feed-forward; capped logits.  Tensor names: ``embed``,
``final.norm``, ``head``, ``l<i>.norm1|norm2``, ``l<i>.hc1|hc2.in|out|mix``, ``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

from ..config.pamazen import PAMAZEN_MODEL_TYPE, AttentionConfig, PamazenConfig
from ..config.registry import register_architecture
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def _rope(rot, head_dim: int) -> dict:
    if rot is None:
        return {"kind": "none"}
    scaling = {"rope_type": "linear", "factor": rot.factor} if rot.factor != 1.0 else None
    return {"kind": "rope", "params": {"head_dim": head_dim, "theta": rot.base, "rotary_dim": rot.dims, "scaling": scaling,
                                       "pairing": "neighbours"}}


def pamazen_model_spec(cfg: PamazenConfig, init_std: float = 0.05) -> ModelSpec:
    W, last = cfg.width, len(cfg.layers) - 1

    def norm(prefix: str) -> PartSpec:
        return PartSpec("rmsnorm", {"size": W, "eps": cfg.norm_eps, "init": ("uniform", 0.8, 1.2), "name": "",
                                    "scalar": True}, prefix)

    def hyper(prefix: str, is_last: bool) -> tuple:
        return ("hyper", PartSpec("hyper_connection", {"hidden_size": W, "streams": cfg.streams, "mult": cfg.residual_mult,
                                                       "last": is_last}, prefix))

    layers, ignored = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        if isinstance(m, AttentionConfig):
            mix = None if not m.v_mix else ("first" if i == cfg.first_value_layer else "mixed")
            if mix != "mixed":              # a file may hold the number of a layer that does not mix
                ignored.append(p + "mix.vmix")
            mixer = PartSpec("softmax_attention", {
                "hidden_size": W, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
                "scale": m.scale, "position": _rope(m.rot, m.dim), "sink": "zero", "value_mix": mix, "init_std": init_std},
                p + "mix.")
        else:
            left, right = m.left, m.right
            mixer = PartSpec("side_by_side", {"hidden_size": W, "mixers": {
                "left": {"kind": "softmax_attention", "scale": m.left_scale, "params": {
                    "hidden_size": W, "num_heads": left.heads, "num_kv_heads": left.kv_heads, "head_dim": left.dim,
                    "value_dim": left.dim, "scale": left.scale, "window": left.window, "keep_first": left.keep_first,
                    "softcap": left.softcap, "sink": "learned", "qk_norm": True, "norm_eps": cfg.norm_eps, "values": "keys",
                    "init_std": init_std}},
                "right": {"kind": "delta_rule", "scale": m.right_scale, "params": {
                    "hidden_size": W, "num_heads": right.heads, "head_dim": right.dim, "norm_eps": cfg.norm_eps,
                    "decay_rank": right.rank, "init_std": init_std}}}}, p + "mix.")
        ff, f = None, layer.mlp
        extra = {"mixer_hyper": hyper(p + "hc1.", i == last and f is None)}
        if f is not None:
            ff = PartSpec("routed_experts", {
                "hidden_size": W, "intermediate_size": f.ff, "num_experts": f.experts, "top": f.top, "gated": True,
                "limit": None, "alpha": 1.0, "up_shift": 0.0, "router": "softmax_top", "renorm": False, "groups": f.groups,
                "keep_groups": f.keep, "identity": f.identity, "shared_ff": f.shared_ff,
                "shared_gate": "shared.sg" if f.shared_ff else None, "init_std": init_std}, p + "mlp.")
            extra["feed_forward_hyper"] = hyper(p + "hc2.", i == last)
        else:                               # no use for a second norm or its connections, whether the file has them or not
            ignored += [p + "norm2", p + "hc2.*"]
        layers.append(LayerSpec(block="hyper", mixer=mixer, feed_forward=ff, mixer_norm=norm(p + "norm1"),
                                feed_forward_norm=norm(p + "norm2") if ff is not None else None, extra=extra))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=W,
        embedding=PartSpec("token", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "embed", "init_std": 1.0}, ""),
        layers=layers, schedule=[ScheduleEntry(i) for i in range(len(layers))], final_norm=norm("final.norm"),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "", "softcap": cfg.logit_softcap,
                                 "init_std": W ** -0.5}, "head"),
        ignored_tensors=tuple(ignored),
    )


register_architecture(PAMAZEN_MODEL_TYPE, PamazenConfig, pamazen_model_spec)
