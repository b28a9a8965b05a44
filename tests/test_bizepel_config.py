"""Bizepel on the host: the registry, config.json's keys, the tensor list, what a request keeps,
which pages a window with kept first tokens gives back, the plain mechanisms against cases made by
hand, error messages."""
import copy
import math

import numpy as np
import pytest

from bizepel_util import (CFG_A, CFG_B, CFG_C, attention_layer, config, delta_layer, dense, file_config, moe, scan_layer,
                          tensor_shapes)
from plain import bizepel_plain as P
from zse_amd import models as _models  # noqa: F401
from zse_amd.cache.manager import CacheManager, GroupInfo, group_needs
from zse_amd.config.base import ConfigError, resolve_architecture
from zse_amd.engine.model import Model
from zse_amd.parts.base import PagedKV, StateNeed


def plan_of(cfg):
    arch = resolve_architecture(cfg)
    return arch.plan(arch.config_from_dict(file_config(cfg)))


def model_of(cfg):
    return Model(plan_of(cfg))


def test_the_architecture_is_found_by_its_name():
    assert resolve_architecture(CFG_A).name == "Bizepel"
    assert resolve_architecture({"model_type": "bizepel"}).name == "Bizepel"


@pytest.mark.parametrize("cfg", [CFG_A, CFG_B, CFG_C])
def test_the_tensor_list_is_the_checkpoints(cfg):
    m = model_of(cfg)
    reqs = {r.name: tuple(r.shape) for r in m.tensor_reqs()}
    want = tensor_shapes(cfg)
    ranks = {f"l{i}.mix.{n}": i for i, l in enumerate(cfg["layers"]) if l["type"] == "general_delta" for n in ("w1", "w2")}
    assert set(reqs) == set(want)
    for n, shape in want.items():
        if n in ranks:          # the rank of the decays' projection is the checkpoint's to say
            assert reqs[n] == ((-1, shape[1]) if n.endswith("w1") else (shape[0], -1))
        else:
            assert reqs[n] == shape, n
    extra = set(tensor_shapes(cfg, unused=True)) - set(want)
    assert extra <= set(m.plan.ignored_tensors)          # the first mixing layer's share may be in the file


def test_what_a_request_keeps():
    m = model_of(CFG_A)
    scan, a1, delta, a2, a3 = m.cache_needs()
    assert isinstance(scan, StateNeed) and scan.nbytes == 4 * (40 * 5 + 3 * 40)
    assert isinstance(delta, StateNeed) and delta.nbytes == 4 * 3 * 12 * 12
    assert isinstance(a1, PagedKV) and (a1.num_kv_heads, a1.head_dim, a1.value_dim, a1.window, a1.keep_first) == (2, 24, 16, 21, 3)
    assert a1.state_bytes == 4 * 3 * (4 * 24 + 2 * 24 + 2 * 16)          # three projected rows of q, k and v
    assert (a2.keep_first, a2.window, a2.state_bytes) == (6, 13, 4 * 2 * (20 + 10 + 14))
    assert (a3.keep_first, a3.window) == (2, 9)
    # both sublayers' input convolutions keep two rows each
    assert m.blocks[0].state_needs() == [("pre_mixer", 4 * 2 * 48), ("pre_ffn", 4 * 2 * 48)]
    assert m.lent == {"values": 32}
    b = model_of(CFG_B)
    assert [k for k, _ in b.blocks[1].state_needs()] == ["pre_mixer"]          # no feed-forward, no second convolution
    assert b.cache_needs()[2].window is None and b.cache_needs()[2].state_bytes == 0
    assert model_of(CFG_C).blocks[0].state_needs() == []                       # one tap looks at nothing earlier
    assert len(group_needs(m.cache_needs())) == 3


def test_every_constant_comes_from_the_config():
    p = plan_of(CFG_A)
    a = p.layers[1].mixer
    assert (a.scale, a.window, a.keep_first, a.conv_taps, a.norm_eps) == (24 ** -0.5, 21, 3, 4, 1e-5)
    assert a.position.interleaved and (a.position.rotary_dim, a.position.theta) == (12, 500.0)
    assert a.lend_values and a.value_share is None
    assert not p.layers[3].mixer.lend_values and p.layers[3].mixer.value_share is None
    assert p.layers[4].mixer.value_share == "l4.mix.vmix" and not p.layers[4].mixer.lend_values
    f = p.layers[1].ffn
    assert (f.scoring, f.gated, f.activation, f.top_k, f.num_experts, f.groups, f.normalise, f.weight_scale) == \
        ("sigmoid", False, "relu2", 3, 6, (3, 2), True, 1.7)
    assert f.correction == "l1.mlp.correction" and f.shared.activation == "relu2" and f.shared.intermediate_size == 40
    assert p.layers[0].ffn.activation == "gelu"
    assert (p.layers[3].side.column, p.layers[3].side.dim, p.layers[3].side.table_columns) == (30, 10, 50)
    assert p.final_norm.gain_scale == 0.5 and p.embedding.norm.weight == "embed.norm" and p.head.weight == "embed"
    assert p.layers[2].filters["pre_ffn"].taps == 3 and p.layers[2].scales == {"mixer": "l2.ls1", "ffn": "l2.ls2"}
    b = plan_of(CFG_B)
    assert b.layers[0].side is None and b.final_norm.gain_scale == 1.0 and b.layers[0].ffn.groups is None
    assert b.layers[0].ffn.shared is None and b.layers[0].ffn.weight_scale == 1.0 and b.layers[1].ffn is None
    assert b.layers[2].mixer.convs is None and b.layers[2].mixer.window is None and b.layers[2].mixer.keep_first == 0
    c = plan_of(CFG_C)
    assert c.layers[1].mixer.position.kind == "none" and c.layers[3].mixer.position.rotary_dim == 2


@pytest.mark.parametrize("window,keep,page", [(21, 3, 4), (8, 9, 4), (5, 1, 8), (40, 16, 16), (1, 0, 4), (7, 20, 4)])
def test_pages_of_the_kept_tokens_stay_and_the_ones_between_go(window, keep, page):
    m = CacheManager([GroupInfo(window, [0], num_pages=64, keep_first=keep)], page_size=page, max_seqs=1, max_model_len=200)
    m.add("r")
    for n in range(1, 190):
        assert m.reserve("r", n)
        m.commit("r", n)
        m.check()
        held = {j for j, p in enumerate(m.table("r", 0)) if p >= 0}
        # what a query at position n or later reads: its window's keys and the kept ones
        need = {j // page for j in range(max(0, n - window + 1), n)} | {j // page for j in range(min(keep, n))}
        assert need <= held, n
        # pages whose every key is out of sight are back in the pool
        assert all((j + 1) * page - 1 >= n - window + 1 or j * page < keep for j in held), n
    m.release("r")
    assert m.pools[0].free_pages == 64


# ---------------------------------------------------------------- the plain mechanisms by hand
def test_plain_visible_keys():
    m = P.visible(8, 3, 2)
    assert m[7].tolist() == [True, True, False, False, False, True, True, True]
    assert m[3].tolist() == [True, True, True, True] + [False] * 4
    assert m[1].tolist() == [True, True] + [False] * 6
    assert P.visible(4, None, 0).sum() == 10


def test_plain_convolution():
    u = np.array([[1.0], [2.0], [4.0], [8.0]])
    assert P.causal_conv(u, np.array([[10.0, 1.0, 0.5]]), np.float64)[:, 0].tolist() == [0.5, 2.0, 14.0, 28.0]


def test_plain_choice_with_groups():
    s = np.array([0.9, 0.1, 0.6, 0.5, 0.8, 0.2])
    # sums of two: 1.0, 1.1, 1.0: the middle group and (the lower number among equals) the first
    assert P.choose(s, np.zeros(6), 2, {"count": 3, "keep": 2}).tolist() == [0, 2]
    # a correction that lifts the last group moves the choice; negative choice scores can win over what is left out
    assert P.choose(s, np.array([0, 0, 0, 0, 0.5, 0.5]), 2, {"count": 3, "keep": 1}).tolist() == [4, 5]
    assert P.choose(s, np.array([-3.0, -3.0, 0, 0, -9, -9]), 3, {"count": 3, "keep": 2}).tolist() == [2, 3, 0]
    assert P.choose(s, np.zeros(6), 2, None).tolist() == [0, 4]


def test_plain_generalized_delta_rule():
    # one channel: u = k / |k|, S <- (w - a) S + k v up to the 1e-6 inside the root
    r, k, v = np.array([[1.0], [2.0]]), np.array([[3.0], [-2.0]]), np.array([[5.0], [7.0]])
    o = P.general_delta_rule(r, k, v, np.array([[0.9], [0.8]]), np.array([[0.3], [0.4]]), np.float64)
    assert o[0, 0] == pytest.approx(15.0) and o[1, 0] == pytest.approx(2 * ((0.8 - 0.4) * 15.0 - 14.0), rel=1e-5)
    # removal along the key empties what an earlier write along the same key left
    k2 = np.array([[1.0, 0.0], [1.0, 0.0]])
    o = P.general_delta_rule(k2, k2, np.array([[4.0, 1.0], [0.0, 0.0]]), np.ones((2, 2)), np.ones((2, 2)), np.float64)
    assert np.abs(o[1]).max() < 1e-5


def test_plain_small_functions():
    assert P.gelu_exact(np.array([1.0]))[0] == pytest.approx(0.8413447460685429)
    assert P.relu_squared(np.array([-2.0, 3.0])).tolist() == [0.0, 9.0]
    x = np.array([[1.0, 2.0, 3.0, 6.0]])
    assert P.layer_norm(x, np.ones(4), 0.5, np.float64)[0, 3] == pytest.approx(3.0 / math.sqrt(3.5 + 0.5))
    y = P.rotate_neighbours(np.array([[[1.0, 0.0, 5.0]]]), [2], np.array([0.25]), np.float64)[0, 0]
    assert y.tolist() == pytest.approx([math.cos(0.5), math.sin(0.5), 5.0])


# ---------------------------------------------------------------- what cannot be served
@pytest.mark.parametrize("change,words", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["canon"].update(taps=0), "canon.taps"),
    (lambda c: c["token_side"].update(dim=0), "token_side.dim"),
    (lambda c: c["layers"][0].update(type="mamba9"), "unknown type"),
    (lambda c: c["layers"][0]["mixer"].update(state=500), "state"),
    (lambda c: c["layers"][1]["mixer"].update(heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=5), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "top"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4), "groups"),
    (lambda c: c["layers"][2]["mlp"]["router"].update(top=3), "groups"),
    (lambda c: c["layers"][2]["mixer"].update(dim=300), "dim"),
    (lambda c: c["layers"][4]["mixer"].update(vdim=12), "value channels"),
    (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "mlp.kind"),
])
def test_errors_say_what_is_wrong(change, words):
    cfg = copy.deepcopy(file_config(CFG_A))
    change(cfg)
    with pytest.raises(ConfigError) as e:
        resolve_architecture(cfg).config_from_dict(cfg)
    assert words in str(e.value)


def test_what_is_absent_does_not_exist():
    cfg = config([attention_layer(rot_dims=0, window=None, conv=None, v_mix=False), delta_layer(), scan_layer(mlp=moe(4, 2, 8, None, None, None))],
                 taps=None, side=None, logit_scale=None)
    m = model_of(cfg)
    assert m.blocks[0].filters == {} and m.blocks[0].side is None and m.blocks[0].mixer.conv is None and m.lent == {}
    assert not any("canon" in r.name or "side" in r.name or "conv" in r.name for r in m.tensor_reqs()
                   if not r.name.startswith("l2.mix"))


def test_flops_count_the_kept_keys():
    far, near = (model_of(config([attention_layer(window=8, keep=k, mlp=dense(8))])) for k in (5, 0))
    assert far.flops([(100, 1)], 0) - near.flops([(100, 1)], 0) == 5 * far.blocks[0].mixer.flops_per_key()
    assert far.flops([(0, 9)], 0) - near.flops([(0, 9)], 0) == 1 * far.blocks[0].mixer.flops_per_key()
    assert far.cache_bytes_read(100, 2) == 13 * (2 * 24 + 2 * 16) * 2
