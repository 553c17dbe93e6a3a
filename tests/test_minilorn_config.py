"""Reading a Minilorn config.json: the parts and constants of every kind of layer, the cache groups (a keys-only
group per window for the compressed rows, keys and values of different sizes), the states of the memories and
the embedding's previous token, what may be absent, errors that name the key at fault, and the cache manager's
bookkeeping of the windowed pages and the embedding's state.  No GPU."""
import json

import pytest

from celeg_amd import native
from celeg_amd.config import ModelSpec

ATT = {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 12, "scale": 0.3, "q_temp": {"coef": 0.2, "every": 50}, "softcap": 20.0}
LAT = {"heads": 5, "dim": 12, "rot_dim": 8, "vdim": 14, "q_rank": 22, "kv_rank": 20, "scale": 0.2, "rot": {"base": 3000.0, "dims": 8},
       "mask": {"size": 21}}
MEM = {"heads": 3, "dim": 6, "vdim": 10, "gate_cap": 12.5}
FF = {"kind": "dense", "ff": 40}
CFG = {"architecture": "Minilorn", "vocab": 99, "width": 48, "norm": {"eps": 3e-5},
       "embedding": {"bigram": {"buckets": 30, "mul_prev": 7, "mul_cur": 11}},
       "layers": [{"type": "latent_attention", "mixer": LAT, "mlp": FF}, {"type": "mlstm", "mixer": MEM, "mlp": None},
                  {"type": "attention", "mixer": ATT, "mlp": FF}, {"type": "latent_attention", "mixer": LAT, "mlp": FF},
                  {"type": "mlstm", "mixer": MEM, "mlp": FF}]}


def test_parts_cache_and_tensors():
    d = native.describe_config(CFG)
    spec = d["spec"]
    assert [s["layer"] for s in spec["order"]] == [0, 1, 2, 3, 4]
    assert spec["embedding"]["params"]["pairs"] == {"buckets": 30, "mul_prev": 7, "mul_cur": 11}
    assert spec["embedding"]["tensors"] == {"table": "embed", "pairs": "bigram"}
    assert spec["head"]["kind"] == "linear_head" and spec["head"]["tensors"] == {"weight": "head"}
    assert spec["final_norm"] == {"kind": "rmsnorm", "params": {"width": 48, "eps": 3e-5}, "tensors": {"weight": "final.norm"}}
    lat, mem, att = spec["layers"][:3]
    assert all(l["arrangement"] == "pre_norm" and l["mixer_norm"]["kind"] == "rmsnorm" for l in spec["layers"])
    m = lat["mixer"]["params"]
    assert lat["mixer"]["kind"] == "latent_attention"
    assert {k: m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale", "window", "eps", "sink", "gate")} == \
        {"heads": 5, "dim": 12, "rot_dim": 8, "vdim": 14, "q_rank": 22, "kv_rank": 20, "scale": 0.2, "window": 21, "eps": 3e-5,
         "sink": False, "gate": False}
    assert m["position"]["params"] == {"theta": 3000.0, "rotary_dim": 8, "head_dim": 8, "pairing": "neighbours"}
    assert lat["ffn"]["kind"] == "mlp" and lat["ffn"]["params"] == {"width": 48, "ff": 40, "activation": "xielu", "bias": False}
    assert mem["mixer"]["kind"] == "matrix_memory" and mem["ffn"]["kind"] == "none"
    assert mem["mixer"]["params"] == {"width": 48, "heads": 3, "dim": 6, "vdim": 10, "gate_cap": 12.5, "eps": 3e-5}
    a = att["mixer"]["params"]
    assert att["mixer"]["kind"] == "biased_attention"
    assert {k: a[k] for k in ("heads", "kv_heads", "head_dim", "v_dim", "scale", "sink", "value_norm", "softcap", "query_temperature", "eps")} == \
        {"heads": 6, "kv_heads": 3, "head_dim": 10, "v_dim": 12, "scale": 0.3, "sink": True, "value_norm": True, "softcap": 20.0,
         "query_temperature": {"coef": 0.2, "every": 50}, "eps": 3e-5}
    groups = [(k["kv_heads"], k["head_dim"], k["v_head_dim"], k["keys_only"], k["window"], k["layers"]) for k in d["cache_layout"]["kv_groups"]]
    assert groups == [(1, 28, 0, True, 21, 2), (3, 10, 12, False, None, 1)]
    states = [(s["step"], s["name"], tuple(s["shape"]), s["dtype"]) for s in d["cache_layout"]["states"]]
    memory = lambda step: [(step, "S", (3, 6, 10), "float32"), (step, "n", (3, 6), "float32"), (step, "m", (3,), "float32")]
    assert states == [(-1, "last", (1,), "int32")] + memory(1) + memory(4)
    names = {e["name"]: e["shape"] for e in d["expected_tensors"]}
    assert names["embed"] == [99, 48] and names["bigram"] == [31, 48] and names["head"] == [99, 48]
    assert names["l0.mix.dq"] == [22, 48] and names["l0.mix.dq.norm"] == [22] and names["l0.mix.uq"] == [100, 22]
    assert names["l0.mix.dkv"] == [28, 48] and names["l0.mix.uk"] == [60, 20] and names["l0.mix.uv"] == [70, 20] and names["l0.mix.o"] == [48, 70]
    assert names["l1.mix.q"] == [18, 48] and names["l1.mix.v"] == [30, 48] and names["l1.mix.i"] == [3, 48] and names["l1.mix.f.b"] == [3]
    assert names["l1.mix.norm"] == [30] and names["l1.mix.o"] == [48, 30]
    assert names["l2.mix.sink"] == [6] and names["l2.mix.v"] == [36, 48] and names["l2.mix.o"] == [48, 72] and names["l2.mlp.act"] == [2]
    assert "l1.norm2" not in names and "l1.mlp.up" not in names and "l0.mix.q" not in names
    again = ModelSpec.from_json(spec).to_json()
    assert again["embedding"] == spec["embedding"] and again["layers"][1] == spec["layers"][1]
    assert d["graph_safe"] is True


def test_what_may_be_absent():
    cfg = json.loads(json.dumps(CFG))
    del cfg["embedding"]
    for key in ("q_temp", "softcap", "vdim", "kv_heads"):
        del cfg["layers"][2]["mixer"][key]
    del cfg["layers"][0]["mixer"]["mask"]
    cfg["layers"][3]["mixer"]["rot_dim"] = 0
    del cfg["layers"][3]["mixer"]["rot"]
    d = native.describe_config(cfg)
    spec = d["spec"]
    assert "pairs" not in spec["embedding"]["params"] and "bigram" not in {e["name"] for e in d["expected_tensors"]}
    assert not [s for s in d["cache_layout"]["states"] if s["step"] == -1]
    a = spec["layers"][2]["mixer"]["params"]
    assert a["kv_heads"] == 6 and a["v_dim"] == 10 and "softcap" not in a and "query_temperature" not in a
    assert "window" not in spec["layers"][0]["mixer"]["params"] and "position" not in spec["layers"][3]["mixer"]["params"]
    assert [(k["head_dim"], k["window"]) for k in d["cache_layout"]["kv_groups"]] == [(28, None), (10, None), (20, 21)]


@pytest.mark.parametrize("path,value,word", [
    (("layers", 1, "type"), "conv", "known types"),
    (("layers", 2, "mixer", "kv_heads"), 4, "multiple of 'kv_heads'"),
    (("layers", 2, "mixer", "softcap"), 0.0, "softcap"),
    (("layers", 2, "mixer", "q_temp", "every"), 0, "q_temp.'every'"),
    (("layers", 2, "mixer", "vdim"), 300, "'vdim' may be at most"),
    (("layers", 0, "mixer", "rot", "dims"), 10, "rot.dims"),
    (("layers", 0, "mixer", "q_rank"), 0, "'q_rank'"),
    (("layers", 0, "mixer", "mask", "size"), 0, "mask.'size'"),
    (("layers", 1, "mixer", "gate_cap"), -1.0, "gate_cap"),
    (("layers", 1, "mixer", "dim"), 300, "'dim' may be at most"),
    (("layers", 1, "mixer", "vdim"), 600, "'vdim' may be at most"),
    (("layers", 0, "mlp", "kind"), "moe", "known kinds"),
    (("layers", 0, "mlp", "ff"), 0, "'ff'"),
    (("embedding", "bigram", "buckets"), 0, "bigram.'buckets'"),
    (("embedding", "bigram", "mul_prev"), 1.5, "bigram.'mul_prev'"),
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


def test_windowed_pages_and_the_embeddings_state():
    """The cache manager's bookkeeping alone: as a request grows, the pages the window has passed go back to the
    pool, the other group keeps all of its own; the embedding's state has a place of its own in every slot."""
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
        assert len(held[0]) == total - max(0, at - n - 21 + 1) // 4
        assert len(held[1]) == total
        cache.call("check")
    cache.call("close", slot)
    assert cache.call("state")["free_pages"] == [40, 40]
