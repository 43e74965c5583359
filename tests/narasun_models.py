"""Small Narasun configurations for the tests and the folders they are written to: random weights made sharp, so that a
misplaced key, a lost or stale state, a forgotten sink, bias or bonus, or a pass that was not given its input moves the
logits by far more than rounding."""
import copy
import json
import math
import os

import torch


def memory(heads, dim, vdim, cap, kind="mlstm"):
    return {"type": kind, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def parallel(left, right, left_scale, right_scale):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def attention(heads, kv_heads, dim, vdim, scale, coef=None, every=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if coef is not None:
        m["q_temp"] = {"coef": coef, "every": every}
    return m


def time_mix(heads, dim, rank):
    return {"heads": heads, "dim": dim, "rank": rank}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def model(vocab, width, eps, layers, loop=None):
    out = {"architecture": "Narasun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CONFIGS = {
    # layers that differ in everything: two pairs of mixers whose head counts, widths and temperatures differ, values wider and
    # narrower than keys, grouped heads, experts of which two are chosen, a layer without feed-forward, two layers that run twice
    "A": model(300, 64, 1e-5, [
        layer(parallel(attention(4, 2, 16, 24, 0.3, 0.5, 16), time_mix(3, 16, 12), 0.8, 1.3), moe(6, 2, 24)),
        layer(memory(4, 16, 24, 8.0), dense(80)),
        layer(parallel(attention(3, 1, 24, 8, 0.25, 0.2, 7), time_mix(2, 24, 5), 1.1, 0.4), moe(5, 3, 32)),
        layer(memory(2, 24, 8, 3.0, "mlstm_2"), None),
        layer(memory(3, 8, 40, 15.0), moe(4, 1, 40)),
    ], loop=(1, 3, 2)),
    # what one model of the design may happen to make equal or 1, made so here and otherwise elsewhere: as many kv heads as
    # heads, values as wide as keys, both factors 1, one head, no temperature, one expert chosen, no loop
    "B": model(131, 88, 1e-6, [
        layer(parallel(attention(3, 3, 12, 12, 0.4), time_mix(1, 12, 3), 1.0, 1.0), moe(4, 1, 40)),
        layer(memory(1, 12, 12, 5.0), dense(56)),
        layer(memory(2, 12, 12, 5.0, "mlstm_2"), moe(3, 1, 24)),
    ]),
    # sizes the matrix-core kernels take, a layer that runs three times, the loop from the first layer
    "C": model(512, 128, 1e-5, [
        layer(memory(4, 64, 64, 12.0), moe(14, 4, 64)),
        layer(parallel(attention(4, 2, 64, 64, 0.11, 0.3, 32), time_mix(4, 64, 32), 0.6, 0.9), dense(256)),
        layer(memory(2, 32, 128, 12.0, "mlstm_2"), moe(8, 2, 64)),
    ], loop=(0, 1, 3)),
    # nothing a multiple of 8; every expert chosen; the whole model in the loop; a temperature that steps at every token
    "D": model(99, 100, 1e-5, [
        layer(memory(3, 10, 14, 4.0), moe(3, 3, 22)),
        layer(parallel(attention(3, 1, 10, 14, 0.6, 0.4, 1), time_mix(3, 10, 6), 1.4, 0.7), None),
        layer(memory(2, 14, 18, 6.0, "mlstm_2"), dense(30)),
    ], loop=(0, 3, 2)),
    # a size at which the products take their other kernels (weights in tiles, K in slices, the library for prompts), heads of
    # 128 channels in the recurrences, many experts
    "E": model(1000, 512, 1e-5, [
        layer(memory(4, 128, 256, 15.0), moe(30, 6, 256)),
        layer(parallel(attention(8, 2, 128, 128, 0.09, 0.2, 100), time_mix(4, 128, 64), 0.7, 0.8), moe(12, 2, 128)),
        layer(memory(8, 32, 64, 15.0, "mlstm_2"), dense(1024)),
        layer(parallel(attention(6, 6, 48, 96, 0.15, 0.5, 50), time_mix(8, 32, 16), 1.2, 0.5), dense(512)),
    ], loop=(1, 3, 2)),
}


def config(name):
    return copy.deepcopy(CONFIGS[name])


def router_values(n):
    """n distinct router logits between -2 and 2.6, unevenly spaced, no two closer than half the mean spacing."""
    step = 4.6 / max(n - 1, 1)
    return [-2.0 + step * k + 0.2 * step * math.sin(1.7 * k + 0.3) for k in range(n)]


def write_model(folder, cfg, seed, gain=1.0, keep_rank=True, decisive_router=False):
    """config.json and model.safetensors with seeded weights, bfloat16-representable, shaped so that faults show: norm weights
    away from one, query/key projections with a gain (peaked attention), sinks of both signs, decays and forget gates from
    forgetting within a few tokens to remembering hundreds, input gates of both signs, a bonus as large as the state's part,
    pass inputs as large as the stream.  Without ``keep_rank`` the written config.json leaves the decays' ranks to the
    tensors' shapes.

    With ``decisive_router`` no choice of experts is a close call, so that an engine that rounds its activations to
    bfloat16 makes the choices of the exact model: output e of a router reads channel e of its input alone, a token's
    embedding holds a permutation of ``router_values`` on those channels, nothing else writes into them, a pass hands them on
    as they are, and the norms before the experts have weight one on them."""
    from safetensors.torch import save_file
    from inferflux_amd.config import config_from_dict
    from inferflux_amd.engine.model import Model
    g = torch.Generator().manual_seed(seed)
    specs = Model.param_specs_for(config_from_dict(cfg))
    tensors = {}
    for name, spec in specs.items():
        shape = tuple(spec.shape)
        if name.endswith((".norm1", "final.norm")):
            t = 0.3 * torch.randn(shape, generator=g)
        elif name.endswith(".norm"):
            t = 1.0 + 0.3 * torch.randn(shape, generator=g)
        elif name.endswith(".sink"):
            t = 1.5 * torch.randn(shape, generator=g)
        elif ".mu." in name:
            t = torch.rand(shape, generator=g)
        elif name.endswith(".w0"):
            t = -6.0 + 7.0 * torch.rand(shape, generator=g)
        elif name.endswith(".u"):
            t = 1.0 + 0.5 * torch.randn(shape, generator=g)
        elif name.endswith(".i.b"):
            t = torch.randn(shape, generator=g)
        elif name.endswith(".f.b"):
            t = -1.0 + 7.0 * torch.rand(shape, generator=g)
        elif name == "loop.step":
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) / (shape[-1] ** 0.5)
            if name.endswith((".left.q", ".left.k")):
                t = t * gain
            elif name.endswith((".mix.i", ".mix.f", ".router")):
                t = t * 2.0
            elif name == "loop.in":
                t = t * 1.5
        tensors[name] = t.to(torch.bfloat16).contiguous()
    # A recurrent head's output is divided by its root mean square.  Queries that lean towards the keys of their own token keep it
    # away from zero, where that division would turn the rounding of one q . k into a large part of the row.
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}.mix"
        q, k = (f"{p}.right.r", f"{p}.right.k") if L["type"] == "parallel" else (f"{p}.q", f"{p}.k")
        tensors[q] = (0.8 * tensors[k].float() + 0.6 * tensors[q].float()).to(torch.bfloat16)
    n = max([L["mlp"]["router"]["experts"] for L in cfg["layers"] if L["mlp"] is not None and L["mlp"]["kind"] == "moe"], default=0)
    if decisive_router and n:
        values = torch.tensor(router_values(n))
        for tok in range(cfg["vocab"]):
            tensors["embed"][tok, :n] = values[torch.randperm(n, generator=g)].to(torch.bfloat16)
        for name, t in tensors.items():
            if name.endswith((".o", ".down")):
                t[:n] = 0
            elif name.endswith(".norm1"):
                t[:n] = 0
            elif name == "loop.step":
                t[:, :n] = 0
            elif name == "loop.in":
                t[:n] = 0
                t[:n, :n] = 0.5 * torch.eye(n).to(t.dtype)
                t[:n, cfg["width"]:cfg["width"] + n] = 0.5 * torch.eye(n).to(t.dtype)
            elif name.endswith(".router"):
                t.zero_()
                t[:, :t.shape[0]] = torch.eye(t.shape[0]).to(t.dtype)
    os.makedirs(folder, exist_ok=True)
    written = copy.deepcopy(cfg)
    if not keep_rank:
        for L in written["layers"]:
            if L["type"] == "parallel":
                L["mixer"]["right"].pop("rank", None)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(written, f)
    save_file(tensors, os.path.join(folder, "model.safetensors"))
    return folder


def load_plain(folder):
    """(config, tensors as float64 arrays) for the plain implementation."""
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    return cfg, {k: v.to(torch.float64).numpy() for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
