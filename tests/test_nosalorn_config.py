"""Reading a Nosalorn config.json: the parts and constants of every kind of layer, which attention layers keep and
which mix their values, the cache groups (per window and kept first keys), the states of the recurrences, what may
be absent, errors that name the key at fault, and the cache manager's bookkeeping of the windowed pages.  No GPU."""
import json

import pytest

from celeg_amd import native
from celeg_amd.config import ModelSpec

ATT = {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 12, "scale": 0.3, "v_mix": True, "mask": {"size": 21, "keep_first": 5},
       "rot": {"base": 3000.0, "dims": 8, "scaling": {"factor": 4.0, "original": 300, "fast": 16.0, "slow": 1.0}}}
LIN = {"heads": 3, "dim": 6, "vdim": 10, "decay": [0.5, 0.9, 1.0]}
SSM = {"heads": 4, "vdim": 14, "state": 9, "groups": 2, "conv": 5, "norm_groups": 7}
FF = {"kind": "dense", "ff": 40}
MOE = {"kind": "moe", "expert": {"ff": 22, "limit": 1.5}, "shared": {"ff": 26, "limit": 0.7},
       "router": {"experts": 7, "top": 3, "scale": 2.5, "identity": 2, "groups": {"count": 3, "keep": 2}}}
CFG = {"architecture": "Nosalorn", "vocab": 99, "width": 48, "norm": {"eps": 3e-5}, "embedding": {"scale": 6.5}, "logit_scale": 0.75,
       "layers": [{"type": "mamba2", "mixer": SSM, "mlp": FF}, {"type": "attention", "mixer": dict(ATT, v_mix=False, mask=None), "mlp": None},
                  {"type": "attention", "mixer": ATT, "mlp": MOE}, {"type": "lightning", "mixer": LIN, "mlp": MOE},
                  {"type": "attention", "mixer": ATT, "mlp": FF}]}


def test_parts_cache_and_tensors():
    d = native.describe_config(CFG)
    spec = d["spec"]
    assert [s["layer"] for s in spec["order"]] == [0, 1, 2, 3, 4]
    assert spec["embedding"]["params"]["scale"] == 6.5 and spec["head"]["params"]["scale"] == 0.75
    assert spec["final_norm"] == {"kind": "rmsnorm", "params": {"width": 48, "eps": 3e-5}, "tensors": {"weight": "final.norm"}}
    assert all(l["arrangement"] == "pre_norm" and l["mixer_norm"]["kind"] == "rmsnorm" for l in spec["layers"])
    ssm, plain_att, keep, lin, mix = spec["layers"]
    assert ssm["mixer"]["kind"] == "state_space" and ssm["ffn"]["kind"] == "swiglu"
    assert ssm["mixer"]["params"] == {"width": 48, "heads": 4, "vdim": 14, "state": 9, "groups": 2, "taps": 5, "norm_groups": 7, "eps": 3e-5}
    assert lin["mixer"]["kind"] == "fixed_decay_attention"
    assert lin["mixer"]["params"] == {"width": 48, "heads": 3, "dim": 6, "vdim": 10, "decay": [0.5, 0.9, 1.0], "eps": 3e-5}
    a = keep["mixer"]["params"]
    assert keep["mixer"]["kind"] == "biased_attention"
    assert {k: a[k] for k in ("heads", "kv_heads", "head_dim", "v_dim", "scale", "bias", "window", "keep_first", "value_mix")} == \
        {"heads": 6, "kv_heads": 3, "head_dim": 10, "v_dim": 12, "scale": 0.3, "bias": True, "window": 21, "keep_first": 5, "value_mix": "keep"}
    assert a["position"]["params"] == {"theta": 3000.0, "rotary_dim": 8, "head_dim": 10, "pairing": "halves",
                                       "scaling": {"rule": "yarn", "factor": 4.0, "original": 300, "fast": 16.0, "slow": 1.0}}
    assert plain_att["mixer"]["params"]["value_mix"] == "none" and "window" not in plain_att["mixer"]["params"]
    assert mix["mixer"]["params"]["value_mix"] == "mix" and mix["mixer"]["tensors"]["mix"] == "l4.mix.vmix"
    f = keep["ffn"]["params"]
    assert keep["ffn"]["kind"] == "routed_experts"
    assert {k: f[k] for k in ("ff", "experts", "identity", "top", "score", "renormalize", "route_scale", "groups", "group_score", "correction",
                              "weight_on", "activation", "limit", "alpha", "shared_gate")} == \
        {"ff": 22, "experts": 7, "identity": 2, "top": 3, "score": "softmax", "renormalize": False, "route_scale": 2.5,
         "groups": {"count": 3, "keep": 2}, "group_score": "best", "correction": True, "weight_on": "output", "activation": "clamped",
         "limit": 1.5, "alpha": 1.702, "shared_gate": True}
    assert f["shared"]["params"] == {"width": 48, "ff": 26, "activation": "clamped", "limit": 0.7, "alpha": 1.702}
    groups = [(k["kv_heads"], k["head_dim"], k["v_head_dim"], k["window"], k["layers"]) for k in d["cache_layout"]["kv_groups"]]
    assert groups == [(3, 10, 12, None, 1), (3, 10, 12, 21, 2)]
    states = [(s["step"], s["name"], tuple(s["shape"]), s["dtype"]) for s in d["cache_layout"]["states"]]
    assert states == [(0, "S", (4, 9, 14), "float32"), (0, "conv", (4, 92), "float32"), (3, "S", (3, 6, 10), "float32")]
    names = {e["name"]: e["shape"] for e in d["expected_tensors"]}
    assert names["l0.mix.in"] == [56 + 92 + 4, 48] and names["l0.mix.conv"] == [92, 5] and names["l0.mix.conv.b"] == [92]
    assert names["l0.mix.A_log"] == names["l0.mix.D"] == names["l0.mix.dt_bias"] == [4] and names["l0.mix.o"] == [48, 56]
    assert names["l2.mix.q.b"] == [60] and names["l2.mix.k.b"] == [30] and names["l2.mix.v.b"] == [36] and names["l4.mix.vmix"] == []
    assert names["l2.mlp.router"] == [9, 48] and names["l2.mlp.correction"] == [9] and names["l2.mlp.e6.gate"] == [22, 48]
    assert names["l2.mlp.shared.sg"] == [1, 48] and names["l2.mlp.shared.down"] == [48, 26]
    assert names["l3.mix.g"] == [30, 48] and names["l3.mix.norm"] == [30] and names["l3.mix.o"] == [48, 30]
    assert "l2.mlp.e7.gate" not in names and "l1.norm2" not in names and "l1.mix.vmix" not in names
    again = ModelSpec.from_json(spec).to_json()
    assert again["layers"] == spec["layers"] and again["embedding"] == spec["embedding"]
    assert d["graph_safe"] is True


def test_what_may_be_absent():
    cfg = json.loads(json.dumps(CFG))
    for key in ("embedding", "logit_scale"):
        del cfg[key]
    att = cfg["layers"][2]["mixer"]
    for key in ("vdim", "kv_heads", "v_mix"):
        del att[key]
    del att["mask"]["keep_first"]
    del att["rot"]["scaling"]
    del cfg["layers"][4]["mixer"]["rot"]
    moe = cfg["layers"][3]["mlp"]
    del moe["shared"]
    for key in ("scale", "identity", "groups"):
        del moe["router"][key]
    del cfg["layers"][3]["mixer"]["vdim"]
    for key in ("groups", "norm_groups"):
        del cfg["layers"][0]["mixer"][key]
    d = native.describe_config(cfg)
    spec = d["spec"]
    assert spec["embedding"]["params"]["scale"] == 1.0 and spec["head"]["params"]["scale"] == 1.0
    a = spec["layers"][2]["mixer"]["params"]
    assert a["kv_heads"] == 6 and a["v_dim"] == 10 and a["value_mix"] == "none" and a["keep_first"] == 0
    assert "scaling" not in a["position"]["params"] and "position" not in spec["layers"][4]["mixer"]["params"]
    assert spec["layers"][4]["mixer"]["params"]["value_mix"] == "keep"       # the first that mixes
    f = spec["layers"][3]["ffn"]["params"]
    assert f["identity"] == 0 and f["groups"] == {"count": 1, "keep": 1} and f["route_scale"] == 1.0 and "shared" not in f
    assert spec["layers"][3]["mixer"]["params"]["vdim"] == 6
    assert spec["layers"][0]["mixer"]["params"]["groups"] == 1 and spec["layers"][0]["mixer"]["params"]["norm_groups"] == 1


@pytest.mark.parametrize("path,value,word", [
    (("layers", 1, "type"), "conv", "known types"),
    (("layers", 2, "mixer", "kv_heads"), 4, "multiple of 'kv_heads'"),
    (("layers", 2, "mixer", "vdim"), 300, "'vdim' may be at most"),
    (("layers", 4, "mixer", "vdim"), 13, "'v_mix'"),
    (("layers", 2, "mixer", "rot", "dims"), 12, "rot.dims"),
    (("layers", 2, "mixer", "rot", "scaling", "factor"), 0.0, "rot.scaling.'factor'"),
    (("layers", 2, "mixer", "mask", "size"), 0, "mask.'size'"),
    (("layers", 2, "mixer", "mask", "keep_first"), -1, "mask.'keep_first'"),
    (("layers", 3, "mixer", "dim"), 300, "'dim' may be at most"),
    (("layers", 3, "mixer", "decay"), [0.5, 0.9], "'decay' must list a number per head"),
    (("layers", 3, "mixer", "decay"), [0.5, 0.9, 1.1], "'decay' holds numbers above 0"),
    (("layers", 0, "mixer", "state"), 300, "'state' may be at most"),
    (("layers", 0, "mixer", "groups"), 3, "multiple of 'groups'"),
    (("layers", 0, "mixer", "norm_groups"), 5, "'norm_groups' must divide"),
    (("layers", 0, "mixer", "conv"), 0, "'conv'"),
    (("layers", 0, "mlp", "kind"), "plain", "known kinds"),
    (("layers", 0, "mlp", "ff"), 0, "'ff'"),
    (("layers", 2, "mlp", "expert", "limit"), 0.0, "expert.'limit'"),
    (("layers", 2, "mlp", "shared", "limit"), -1.0, "shared.'limit'"),
    (("layers", 2, "mlp", "router", "top"), 10, "'top' exceeds"),
    (("layers", 2, "mlp", "router", "top"), 7, "fewer experts than 'top'"),
    (("layers", 2, "mlp", "router", "groups", "count"), 4, "'groups.count'"),
    (("layers", 2, "mlp", "router", "identity"), -1, "'identity'"),
    (("norm", "eps"), 0.0, "norm.eps"),
])
def test_errors_name_the_key(path, value, word):
    cfg = json.loads(json.dumps(CFG))
    at = cfg
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(native.NativeArgumentError) as err:
        native.describe_config(cfg)
    assert word in str(err.value), str(err.value)


def test_windowed_pages_and_kept_first_ones():
    """The cache manager's bookkeeping alone: as a request grows, the pages the window has passed go back to the pool,
    but for those of the kept first keys; the other group keeps all of its own."""
    layout = native.describe_config(CFG)["cache_layout"]
    cache = native.HostObject("cache", layout=layout, page_tokens=4, n_pages=[40, 40], max_requests=2, max_context=160)
    slot = cache.call("open")
    at = 0
    for n in (30, 1, 1, 17, 2, 40):
        assert cache.call("prepare", slot, at, n)
        at += n
        assert cache.call("covers", slot, at - n, n)
        held = cache.call("pages_held", slot)
        total = (at + 3) // 4
        assert len(held[0]) == total
        assert len(held[1]) == total - max(0, max(0, at - n - 21 + 1) // 4 - 2)      # five kept keys lie in two pages
        cache.call("check")
    cache.call("close", slot)
    assert cache.call("state")["free_pages"] == [40, 40]
