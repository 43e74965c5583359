"""The Narasun decoder as a plan of parts.

A token's row of ``embed`` starts the residual stream.  Every layer has one RMS norm, whose weight is stored as the difference
from one, and both of the layer's sub-blocks read its output: x <- x + mixer(norm1(x)) + ff(norm1(x)).  After the last layer
the model's norm (``final.norm``) and an output matrix of its own (``head``) follow.  A layer's mixer is one of

  parallel           two mixers over the same rows whose outputs are added with a factor each: softmax attention without
                     positions, whose queries grow with the logarithm of their position and whose denominator holds a learned
                     sink per head; and time mixing, a matrix state per head with a decay per key channel and token and a
                     bonus for the current token, fed by mixes of each row with the row before it
  mlstm, mlstm_2     matrix memory with exponential input and forget gates, a normaliser and a running maximum

and its feed-forward a gated one or a mixture of experts whose router takes a sigmoid and whose weights multiply the experts'
inputs.  A span of layers may run several times in a row (``loop``): the schedule names those layers once per pass, which gives
each pass its own cache and state, and the first layer of each pass is preceded by that pass's input, which replaces the
stream by a matrix times [stream; embedding] plus the pass's row of ``loop.step``.

Tensor names: ``embed``, ``head``, ``loop.in``, ``loop.step``, ``l<i>.norm1``, ``l<i>.mix.*`` (``.left.*`` and ``.right.*`` for
two mixers), ``l<i>.mlp.*``, ``final.norm``; a bias is its matrix's name with ``.b``.
"""
from __future__ import annotations

from ..config.base import ConfigError
from ..config.narasun import NarasunConfig
from ..config.registry import register_architecture
from ..parts.plan import LayerSpec, ModelPlan, PartSpec, ScheduleEntry


def _attention(p: str, m) -> PartSpec:
    names = {k: f"{p}.{k}" for k in ("q", "k", "v", "o", "sink")}
    return PartSpec("paged_attention", {
        "name": p, "n_heads": m.heads, "n_kv_heads": m.kv_heads, "head_dim": m.dim, "v_head_dim": m.vdim, "bias": False,
        "scale": m.scale, "sinks": True, "q_temp": m.q_temp.to_dict() if m.q_temp is not None else None,
        "position": PartSpec("none", {}), "tensors": names})


def _time_mix(p: str, i: int, m, cfg: NarasunConfig) -> PartSpec:
    if m.rank is None:
        raise ConfigError(f"config.json: 'layers[{i}].mixer.right.rank' is left to the model file's tensors: load the config from "
                          "a model folder, or name the rank")
    names = {k: f"{p}.{k}" for k in ("r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o")}
    names.update({f"mu_{s}": f"{p}.mu.{s}" for s in "rkvgw"})
    return PartSpec("time_mix", {"name": p, "n_heads": m.heads, "head_dim": m.dim, "decay_rank": m.rank, "norm_eps": cfg.norm_eps,
                                 "tensors": names})


def _matrix_memory(p: str, m, cfg: NarasunConfig) -> PartSpec:
    names = {k: f"{p}.{k}" for k in ("q", "k", "v", "g", "i", "f", "o", "norm")}
    names.update({"i_bias": f"{p}.i.b", "f_bias": f"{p}.f.b"})
    return PartSpec("matrix_memory", {"name": p, "n_heads": m.heads, "head_dim": m.dim, "v_head_dim": m.vdim, "gate_cap": m.gate_cap,
                                      "norm_eps": cfg.norm_eps, "tensors": names})


def _mlp(p: str, m) -> PartSpec:
    if m.kind == "dense":
        return PartSpec("gated_ffn", {"name": p, "intermediate_size": m.ff, "activation": "silu",
                                      "tensors": {k: f"{p}.{k}" for k in ("gate", "up", "down")}})
    return PartSpec("moe", {"name": p, "n_experts": m.experts, "top": m.top, "ff": m.ff, "scoring": "sigmoid", "renormalize": False,
                            "weigh_input": True})


def narasun_plan(cfg: NarasunConfig) -> ModelPlan:
    layers = []
    norm = lambda name: PartSpec("rmsnorm", {"name": name, "tensor": name, "eps": cfg.norm_eps, "offset": 1.0})
    for i, L in enumerate(cfg.layers):
        p = f"l{i}"
        if L.type == "parallel":
            mixer = PartSpec("side_by_side", {
                "name": f"{p}.mix", "mixers": (_attention(f"{p}.mix.left", L.mixer.left), _time_mix(f"{p}.mix.right", i, L.mixer.right, cfg)),
                "scales": (L.mixer.left_scale, L.mixer.right_scale)})
        else:
            mixer = _matrix_memory(f"{p}.mix", L.mixer, cfg)
        layers.append(LayerSpec(prefix=p, block=PartSpec("parallel", {}), norm_in=norm(f"{p}.norm1"), mixer=mixer,
                                ffn=_mlp(f"{p}.mlp", L.mlp) if L.mlp is not None else None))
    times = cfg.loop.times if cfg.loop is not None else 0
    injections = tuple(PartSpec("projected_pass_input", {"index": t, "times": times, "matrix": "loop.in", "tensor": "loop.step"})
                       for t in range(times))
    return ModelPlan(
        vocab_size=cfg.vocab, hidden_size=cfg.width, max_position=cfg.max_positions,
        embedding=PartSpec("token_embedding", {"name": "embed", "tensor": "embed", "vocab_size": cfg.vocab}),
        layers=tuple(layers), schedule=tuple(ScheduleEntry(i, before=t) for i, t in cfg.run_order()),
        final_norm=norm("final.norm"),
        lm_head=PartSpec("linear_head", {"name": "head", "tensor": "head", "vocab_size": cfg.vocab}),
        injections=injections,
    )


register_architecture(NarasunConfig, narasun_plan)
