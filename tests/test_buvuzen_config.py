"""Buvuzen on the host: the registry, config.json's keys, the tensor list, layers with the weights of
another one, what a request keeps, the plain mechanisms against cases made by hand, error messages."""
import copy

import numpy as np
import pytest

from buvuzen_util import CFG_A, CFG_B, CFG_C, again, config, layer, moe, random_weights, tensor_shapes
from plain import buvuzen_plain as P
from zse_amd import models as _models  # noqa: F401
from zse_amd.config.base import ConfigError, resolve_architecture
from zse_amd.engine.model import Model
from zse_amd.parts.base import PagedKV


def plan_of(cfg):
    arch = resolve_architecture(cfg)
    return arch.plan(arch.config_from_dict(cfg))


def test_the_architecture_is_found_by_its_name():
    assert resolve_architecture(CFG_A).name == "Buvuzen"
    assert resolve_architecture({"model_type": "buvuzen"}).name == "Buvuzen"


@pytest.mark.parametrize("cfg", [CFG_A, CFG_B, CFG_C])
def test_the_tensor_list_is_the_checkpoints(cfg):
    reqs = {r.name: tuple(r.shape) for r in Model(plan_of(cfg)).tensor_reqs()}
    assert reqs == tensor_shapes(cfg)


def test_layers_that_use_anothers_weights_keep_keys_of_their_own():
    plan = plan_of(CFG_A)
    assert [c.layer for c in plan.order] == [0, 1, 2, 0, 1, 0] and len(plan.layers) == 3
    assert all(c.cache_of is None for c in plan.order)
    m = Model(plan)
    needs = m.cache_needs()
    assert all(isinstance(n, PagedKV) for n in needs) and len(needs) == 6
    assert [(n.num_kv_heads, n.head_dim, n.value_dim, n.window) for n in needs[:3]] == [(2, 24, 20, 13), (3, 20, 28, 29), (1, 12, None, None)]
    assert needs[3] == needs[5] == needs[0] and needs[4] == needs[1]
    # a layer may come before the one whose weights it uses, and name one that names another
    c = plan_of(CFG_C)
    assert [x.layer for x in c.order] == [1, 0, 1] and [b.mixer.names["q"] for b in c.layers] == ["l1.mix.q", "l2.mix.q"]
    chain = copy.deepcopy(CFG_A)
    chain["layers"][5]["weights_of"] = 3
    assert [x.layer for x in plan_of(chain).order] == [0, 1, 2, 0, 1, 0]


def test_every_constant_comes_from_the_config():
    plan = plan_of(CFG_A)
    b = plan.layers[0]
    assert b.arrangement == "postnorm" and set(b.norms) == {"post_mixer", "post_ffn"}
    assert b.norms["post_mixer"].unit_offset and b.norms["post_mixer"].eps == 1e-5
    a = b.mixer
    assert (a.scale, a.window, a.value_dim, a.softcap, a.norm_eps) == (24 ** -0.5, 13, 20, None, 1e-5)
    assert (a.sinks, a.head_gate, a.q_norm, a.position.kind) == ("l0.mix.sink", "l0.mix.g", "l0.mix.q.norm", "none")
    f = b.ffn
    assert (f.num_experts, f.identity, f.top_k, f.groups, f.group_best, f.weight_scale) == (7, 2, 3, (3, 2), 1, 2.2)
    assert (f.scoring, f.scale_input, f.activation, f.normalise) == ("softmax", False, "silu", False)
    assert f.shared_gate == "l0.mlp.shared.sg" and f.shared.intermediate_size == 40
    assert plan.layers[1].ffn is None and set(plan.layers[1].norms) == {"post_mixer"}
    assert plan.layers[2].mixer.window is None and plan.layers[2].ffn.groups is None
    assert plan_of(CFG_B).layers[1].ffn.shared is None and plan_of(CFG_B).layers[1].ffn.identity == 0
    assert plan.embedding.scale == 5.3 and plan.final_norm.gain_scale == 0.7 and plan.head.weight == "head"


def test_the_embeddings_scale_is_not_rounded():
    """5.3 is no bfloat16 number; the stream is a 32-bit one from the start."""
    from zse_amd.parts.embedding import Embedding

    class Source:
        def matrix(self, names, strip=False):
            return None

    e = Embedding(plan_of(CFG_A).embedding)
    e.load(Source(), None, "bfloat16")
    assert e.scale == float(np.float32(5.3))


def test_plain_mechanisms_against_cases_made_by_hand():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(P.model_norm(x, np.array([0.0, 1.0]), 0.0, np.float64), x / np.sqrt(12.5) * [1.0, 2.0])
    assert np.allclose(P.head_norm(x, np.array([2.0, 3.0]), 0.0, np.float64), x / np.sqrt(12.5) * [2.0, 3.0])
    # a window of 3 sees itself and two tokens before it
    assert P.visible(5, 3)[4].tolist() == [False, False, True, True, True]
    # a sink takes its share of the softmax and gives nothing for it; it counts once and is not scaled
    p = P.sink_softmax(np.log(np.array([[1.0, 2.0, 5.0]])), np.array([[True, True, False]]), np.log(4.0))
    assert np.allclose(p, [[1 / 7, 2 / 7, 0.0]])
    # groups: [0 .9 | .5 .6 | -.3 -.2] -- by their best the first group wins, by sums of two the second would
    c = np.array([0.0, 0.9, 0.5, 0.6, -0.3, -0.2])
    assert P.choose(c, 2, (3, 1))[0].tolist() == [1, 0]
    assert P.choose(c, 2, (3, 2))[0].tolist() == [1, 3]
    assert P.choose(c, 2, None)[0].tolist() == [1, 3]
    # choice scores below zero: what is out of the race never wins against what is in it
    assert P.choose(np.array([-0.5, -0.9, -0.6, -0.7]), 2, (2, 1))[0].tolist() == [0, 1]
    assert P.choose(np.array([0.2, 0.2, 0.2]), 2, None)[0].tolist() == [0, 1]
    # an identity expert gives its input back, times its score and the router's scale
    ml = moe(1, 1, 4, None, identity=1, scale=3.0, groups=None)
    w = {"r.router": np.array([[0.0, 0.0], [1.0, 0.0]]), "r.correction": np.array([0.0, 0.0])}
    h = np.array([[2.0, -1.0]])
    s = np.exp(2.0) / (1.0 + np.exp(2.0))
    assert np.allclose(P.mixture(ml, w, "r.", h, np.float64), 3.0 * s * h)
    # the correction counts in the choice alone
    w["r.correction"] = np.array([2.0, 0.0])
    w.update({"r.e0.gate": np.ones((4, 2)), "r.e0.up": np.ones((4, 2)), "r.e0.down": np.ones((2, 4))})
    one = 4 * P.silu(1.0) * 1.0
    assert np.allclose(P.mixture(ml, w, "r.", h, np.float64), 3.0 * (1.0 - s) * one)


def test_the_plain_run_uses_the_weights_a_layer_names():
    cfg = config(again([layer(mlp=moe())], 0))
    w = random_weights(cfg, 1)
    twice = dict(w)
    other = copy.deepcopy(cfg)
    other["layers"][1].pop("weights_of")
    twice.update({n.replace("l0.", "l1."): a for n, a in w.items() if n.startswith("l0.")})
    toks = [5, 9, 1, 1, 60, 3]
    assert np.array_equal(P.forward(cfg, w, toks), P.forward(other, twice, toks))


def test_errors_name_the_layer_and_the_key():
    bad = copy.deepcopy(CFG_A)
    bad["layers"][0]["mixer"]["kv_heads"] = 4
    bad["layers"][1]["mixer"].pop("scale")
    bad["layers"][2]["type"] = "conv"
    with pytest.raises(ConfigError) as e:
        resolve_architecture(bad).config_from_dict(bad)
    msg = str(e.value)
    assert "layer 0" in msg and "kv_heads" in msg and "layer 1" in msg and "'scale'" in msg and "layer 2" in msg and "conv" in msg
    for key in ("vocab", "width", "norm", "layers"):
        c = copy.deepcopy(CFG_B)
        c.pop(key)
        with pytest.raises(ConfigError, match=key):
            resolve_architecture(CFG_B).config_from_dict(c)
    for change, word in ((("router", "top", 10), "top"), (("router", "identity", 1), "groups"), (("router", "identity", -1), "identity"),
                         (("expert", "ff", 0), "ff")):
        c = copy.deepcopy(CFG_A)
        c["layers"][0]["mlp"][change[0]][change[1]] = change[2]
        with pytest.raises(ConfigError, match=word):
            resolve_architecture(c).config_from_dict(c)
    for of in (9, -1, 3):
        c = copy.deepcopy(CFG_A)
        c["layers"][3]["weights_of"] = of
        with pytest.raises(ConfigError, match="weights_of"):
            resolve_architecture(c).config_from_dict(c)
    c = copy.deepcopy(CFG_A)
    c["layers"][3]["mixer"]["heads"] = 2
    with pytest.raises(ConfigError, match="must equal"):
        resolve_architecture(c).config_from_dict(c)


def test_other_orders_can_be_put_together():
    cfg = config([layer(mlp=None), layer(window=1, mlp=moe(2, 1, 8, None, identity=0, groups=None))])
    cfg.pop("embedding")
    cfg.pop("logit_scale")
    plan = plan_of(cfg)
    assert plan.embedding.scale == 1.0 and plan.final_norm.gain_scale == 1.0
    m = Model(plan)
    assert m.blocks[0].ffn is None and m.blocks[1].ffn.choices == 2
