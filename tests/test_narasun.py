"""The Narasun design without a GPU: its config and plan, what the cache and state managers are asked for, and the plain
implementation's mechanisms against closed forms."""
import copy
import json
import math
import os

import numpy as np
import pytest
import torch

import narasun_models as nm
import plain_narasun as pn
from inferflux_amd.cache.storage import plan_groups
from inferflux_amd.config import ConfigError, NarasunConfig, config_from_dict, load_config
from inferflux_amd.engine.model import Model
from inferflux_amd.kernels.ops import DeltaSum, ScaledDelta


def test_config_reads_every_size_and_keeps_absent_keys_meaning():
    cfg = config_from_dict(nm.config("A"))
    assert isinstance(cfg, NarasunConfig) and cfg.vocab == 300 and cfg.width == 64 and cfg.norm_eps == 1e-5
    p, m = cfg.layers[0].mixer, cfg.layers[1].mixer
    assert (p.left.heads, p.left.kv_heads, p.left.dim, p.left.vdim, p.left.scale) == (4, 2, 16, 24, 0.3)
    assert (p.left.q_temp.coef, p.left.q_temp.every, p.left_scale, p.right_scale) == (0.5, 16, 0.8, 1.3)
    assert (p.right.heads, p.right.dim, p.right.rank) == (3, 16, 12)
    assert (m.heads, m.dim, m.vdim, m.gate_cap) == (4, 16, 24, 8.0)
    assert [L.type for L in cfg.layers] == ["parallel", "mlstm", "parallel", "mlstm_2", "mlstm"]
    assert cfg.layers[1].mlp.kind == "dense" and cfg.layers[1].mlp.ff == 80 and cfg.layers[3].mlp is None
    assert (cfg.layers[2].mlp.experts, cfg.layers[2].mlp.top, cfg.layers[2].mlp.ff) == (5, 3, 32)
    assert config_from_dict(cfg.to_dict()) == cfg
    raw = nm.config("B")
    raw["layers"][0]["mixer"]["left"].pop("kv_heads")
    raw["layers"][0]["mixer"]["left"].pop("vdim")
    raw["layers"][1]["mixer"].pop("vdim")
    assert config_from_dict(raw) == config_from_dict(nm.config("B"))
    assert config_from_dict(raw).layers[0].mixer.left.q_temp is None and config_from_dict(raw).loop is None


@pytest.mark.parametrize("path,value,says", [
    (("layers", 0, "mixer", "left", "heads"), 5, "layers[0].mixer.left.heads"), (("layers", 0, "mixer", "left", "q_temp", "every"), 0, "q_temp.every"),
    (("layers", 0, "mixer", "right", "rank"), 0, "layers[0].mixer.right.rank"), (("layers", 2, "type"), "conv", "layers[2].type"),
    (("layers", 0, "mlp", "router", "top"), 9, "layers[0].mlp.router.top"), (("loop", "stop"), 9, "loop"), (("loop", "times"), 0, "loop.times"),
    (("layers", 1, "mixer", "gate_cap"), 0.0, "layers[1].mixer.gate_cap"), (("layers", 3, "mixer", "dim"), "x", "layers[3].mixer.dim"),
    (("layers", 2, "mixer", "left_scale"), None, "layers[2].mixer.left_scale"), (("layers", 2, "mixer", "right"), 4, "layers[2].mixer.right"),
    (("norm", "eps"), -1.0, "norm.eps"), (("layers", 0, "mlp", "kind"), "glu", "layers[0].mlp.kind"),
    (("layers", 0, "mlp", "shared"), {"ff": 8}, "layers[0].mlp.shared")])
def test_config_errors_name_the_key(path, value, says):
    raw = nm.config("A")
    at = raw
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ConfigError) as e:
        config_from_dict(raw)
    assert says in str(e.value)


def test_plan_passes_have_their_own_cache_state_and_input():
    model = Model(config_from_dict(nm.config("A")))
    plan = model.plan
    assert [(e.layer, e.before) for e in plan.schedule] == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]
    assert [j.index for j in model.injections] == [0, 1] and all(j.needs_embedding for j in model.injections)
    mixers = model.schedule_mixers()
    groups, _ = plan_groups(plan.schedule, mixers)
    assert len(groups) == 1 and groups[0].window is None and groups[0].entries == (0, 2, 4)      # each pass its own pages
    assert [m.state_spec() is not None for m in mixers] == [True] * 7
    assert (mixers[0].cache_spec().head_dim, mixers[0].cache_spec().v_dim, mixers[0].cache_spec().n_kv_heads) == (16, 24, 2)
    assert mixers[1].cache_spec() is None and mixers[1].state_spec().shape[0] == 4 + 4 * 25 * 16      # maxima, then values and the normaliser
    assert mixers[0].state_spec().shape[0] == 64 + 3 * 16 * 16                                        # the last row, then S
    specs = model.param_specs()
    assert specs["loop.in"].shape == (64, 128) and specs["loop.step"].shape == (2, 64) and specs["head"].shape == (300, 64)
    assert specs["l0.mix.left.sink"].shape == (4,) and specs["l0.mix.right.u"].shape == (3, 16) and specs["l0.mix.right.w1"].shape == (12, 64)
    assert specs["l1.mix.i.b"].shape == (4,) and specs["l1.mix.norm"].shape == (96,) and "l0.norm2" not in specs
    assert model.graph_safe
    no_loop = Model(config_from_dict(nm.config("B")))
    assert not no_loop.injections and all(e.before is None for e in no_loop.plan.schedule)


def test_rank_left_to_the_tensors(tmp_path):
    folder = nm.write_model(str(tmp_path / "m"), nm.config("A"), 1, keep_rank=False)
    raw = json.load(open(os.path.join(folder, "config.json")))
    assert "rank" not in raw["layers"][0]["mixer"]["right"]
    assert config_from_dict(raw).open_sizes() == ("layers[0].mixer.right.rank", "layers[2].mixer.right.rank")
    with pytest.raises(ConfigError):
        Model(config_from_dict(raw))
    assert [load_config(folder).layers[i].mixer.right.rank for i in (0, 2)] == [12, 5]


def test_sums_of_additions_are_taken_apart():
    a, b, v = torch.ones(2, 3), torch.full((2, 3), 2.0), torch.tensor([1.0, 2.0, 3.0])
    s = DeltaSum([(DeltaSum([(a, 0.5), (ScaledDelta(b, 3.0), 2.0)]), 2.0), (v, 1.0)])
    assert [t[1] for t in s.terms] == [1.0, 12.0, 1.0]
    assert torch.equal(s.tensor(a), a + 12.0 * b + v) and DeltaSum.of(None, a).terms == [(a, 1.0)]


# ---- the plain mechanisms against closed forms ---------------------------------------------------
def test_query_temperature_steps_where_it_should():
    f = pn.query_temperature(40, {"coef": 0.5, "every": 16})
    assert np.all(f[:15] == 1.0) and np.allclose(f[15:31], 1 + 0.5 * math.log(2)) and np.allclose(f[31:], 1 + 0.5 * math.log(3))
    assert np.all(pn.query_temperature(5, None) == 1.0)


def test_sink_takes_its_share_of_the_softmax():
    p = pn.causal_softmax(np.zeros((3, 3)), 0.0)
    assert np.allclose(p, [[1 / 2, 0, 0], [1 / 3, 1 / 3, 0], [1 / 4, 1 / 4, 1 / 4]])
    assert np.allclose(pn.causal_softmax(np.zeros((1, 1)), math.log(4.0)), 0.2)


def test_time_mix_reads_its_own_write_through_the_bonus_alone():
    k, v, w = np.eye(3)[[0, 1, 0]], np.array([[1.0, 2, 3], [4, 5, 6], [7, 8, 9]]), np.full((3, 3), 0.5)
    r = np.eye(3)[[0, 0, 0]]
    u = np.array([2.0, 0, 0])
    out = pn.time_mix_recurrence(r, k, v, w, u)
    assert np.allclose(out[0], 2 * v[0])                       # nothing but the bonus
    assert np.allclose(out[1], v[0])                           # written a token ago, not decayed yet
    assert np.allclose(out[2], 0.5 * v[0] + 2 * v[2])          # decayed once, and the own write through the bonus
    m = pn.shifted_mix(np.array([[1.0], [3.0]]), np.array([0.25]))
    assert np.allclose(m, [[0.75], [2.5]])                     # zeros before the first row


def test_matrix_memory_against_its_unstabilised_form():
    g = np.random.default_rng(3)
    T, d, dv = 30, 5, 4
    q, k, v = g.normal(size=(T, d)), g.normal(size=(T, d)), g.normal(size=(T, dv))
    li, lf = g.normal(size=T) * 2, pn.log_sigmoid(g.normal(size=T))
    out = pn.matrix_memory_recurrence(q, k, v, li, lf)
    S, n = np.zeros((d, dv)), np.zeros(d)
    m, M = 0.0, 0.0
    for t in range(T):                      # without the maximum; the floor exp(-m) becomes 1, the small number exp(m) times itself
        S = np.exp(lf[t]) * S + np.exp(li[t]) * np.outer(k[t], v[t])
        n = np.exp(lf[t]) * n + np.exp(li[t]) * k[t]
        m = max(lf[t] + m, li[t])
        assert np.allclose(out[t], (S.T @ q[t]) / (max(abs(n @ q[t]), 1.0) + 1e-6 * np.exp(m)))
    big = pn.matrix_memory_recurrence(q, k, v, li + 300.0, lf)      # far beyond what an exponential holds
    assert np.all(np.isfinite(big))


def test_weights_on_the_experts_inputs():
    W = {"m.router": np.array([[1.0, 0], [0.0, 0]]), "m.e0.gate": np.eye(2), "m.e0.up": np.eye(2), "m.e0.down": np.eye(2),
         "m.e1.gate": np.eye(2), "m.e1.up": np.eye(2), "m.e1.down": np.eye(2)}
    h = np.array([[2.0, -1.0]])
    s = pn.sigmoid(2.0)
    assert np.allclose(pn.moe(h, W, "m", {"router": {"experts": 2, "top": 1}}), pn.silu(s * h) * s * h)
    both = pn.moe(h, W, "m", {"router": {"experts": 2, "top": 2}})
    assert np.allclose(both, pn.silu(s * h) * s * h + pn.silu(0.5 * h) * 0.5 * h)


def test_every_mechanism_moves_the_logits(tmp_path):
    """Leaving any one mechanism out of the plain model changes its logits by far more than rounding."""
    folder = nm.write_model(str(tmp_path / "m"), nm.config("A"), 5, gain=2.0)
    cfg, W = nm.load_plain(folder)
    ids = torch.randint(0, 300, (70,), generator=torch.Generator().manual_seed(1)).tolist()
    base = pn.forward(cfg, W, ids)

    def moved(change_cfg=None, change_w=None):
        c, w = copy.deepcopy(cfg), dict(W)
        if change_cfg:
            change_cfg(c)
        if change_w:
            change_w(w)
        out = pn.forward(c, w, ids)
        return float(np.abs(out - base).max() / np.abs(base).max())

    def setter(path, value):
        def f(c):
            at = c
            for k in path[:-1]:
                at = at[k]
            at[path[-1]] = value
        return f

    assert moved() == 0.0
    changes = {
        "temperature one later": setter(("layers", 0, "mixer", "left", "q_temp", "every"), 17),
        "temperature's size": setter(("layers", 2, "mixer", "left", "q_temp", "coef"), 0.0), "passes": setter(("loop", "times"), 1),
        "left factor": setter(("layers", 0, "mixer", "left_scale"), 1.0), "right factor": setter(("layers", 2, "mixer", "right_scale"), 1.0),
        "gates' cap": setter(("layers", 3, "mixer", "gate_cap"), 8.0), "scores' factor": setter(("layers", 0, "mixer", "left", "scale"), 0.25),
        "no feed-forward": setter(("layers", 1, "mlp"), None), "one expert fewer": setter(("layers", 2, "mlp", "router", "top"), 2),
    }
    for what, f in changes.items():
        assert moved(change_cfg=f) > 1e-3, what
    zero = lambda name: (lambda w: w.__setitem__(name, np.zeros_like(w[name])))
    for name in ("l0.mix.left.sink", "l0.mix.right.u", "l0.mix.right.w0", "l0.mix.right.w1", "l0.mix.right.mu.g", "l2.mix.right.mu.w", "l1.mix.i.b",
                 "l1.mix.f.b", "loop.step", "l3.norm1", "final.norm"):
        assert moved(change_w=zero(name)) > 1e-3, name
    halves = W["loop.in"].copy()
    halves[:, 64:] = 0.0
    assert moved(change_w=lambda w: w.__setitem__("loop.in", halves)) > 1e-3
