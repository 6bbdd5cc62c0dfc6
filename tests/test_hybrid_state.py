"""State slots, session reuse, the checkpoint reader and the registry."""

import json
import struct

import pytest
import torch

from hybrid_cases import write_checkpoint
from koridra_cases import CONFIGS, RANKS, random_weights
from quoracle_amd.engine.kv_cache import (BlockManager, OutOfBlocks,
                                          OutOfSlots, SessionCache, StateSlots)
from quoracle_amd.models import KoridraModel, build_model, get_config
from quoracle_amd.models.checkpoint import Checkpoint
from quoracle_amd.models.hybrid_config import KoridraConfig


def sessions(blocks=8, slots=2):
    return SessionCache(BlockManager(blocks, 4), StateSlots(slots))


def test_slots_are_given_and_given_back():
    c = sessions()
    a, b, d = (c.get_or_create(x) for x in "abd")
    c.extend(a, [1, 2])
    c.extend(b, [1])
    assert {a.state_slot, b.state_slot} == {0, 1}
    with pytest.raises(OutOfSlots):
        c.extend(d, [1], active=["a", "b", "d"])
    assert not c.place(d, ["a", "b", "d"])
    held = a.state_slot
    c.drop("a")
    assert a.state_slot == -1 and c.place(d, ["b", "d"])
    assert d.state_slot == held


def test_idle_session_is_evicted_for_a_slot():
    c = sessions()
    a, b, d = (c.get_or_create(x) for x in "abd")
    c.extend(a, [1])
    c.extend(b, [1])
    assert c.place(d, ["b", "d"])          # a is idle
    assert a.state_slot == -1 and a.blocks == []


def test_out_of_slots_is_a_full_cache():
    assert issubclass(OutOfSlots, OutOfBlocks)


def test_state_reuse_is_all_or_nothing():
    c = sessions()
    a = c.get_or_create("a")
    c.extend(a, [1, 2, 3, 4, 5])
    assert c.match_prefix(a, [1, 2, 3, 4, 5, 6]) == 5
    assert c.match_prefix(a, [1, 2, 3, 9]) == 0
    assert a.token_ids == [] and a.blocks == [] and a.state_slot >= 0
    assert c.mgr.free_blocks == 8


def test_last_prompt_token_is_never_cached():
    """Its logits are needed, with and without a recurrent state."""
    c = sessions()
    a = c.get_or_create("a")
    c.extend(a, [1, 2, 3])
    assert c.match_prefix(a, [1, 2, 3]) == 0
    plain = SessionCache(BlockManager(8, 4))
    b = plain.get_or_create("b")
    plain.extend(b, [1, 2, 3])
    assert plain.match_prefix(b, [1, 2, 3]) == 2


def test_checkpoint_reader(tmp_path):
    cfg = CONFIGS["odd"]
    w = random_weights(cfg, RANKS["odd"])
    folder = write_checkpoint(str(tmp_path / "m"), cfg, w)
    c = Checkpoint(folder + "/model.safetensors")
    assert set(c.names()) == set(w)
    for name, t in w.items():
        assert c.shape(name) == tuple(t.shape)
        assert torch.equal(c.get(name), t)
    with pytest.raises(KeyError):
        c.get("nothing")
    bad = tmp_path / "bad.safetensors"
    bad.write_bytes(struct.pack("<Q", 1 << 40) + b"{}")
    with pytest.raises(ValueError):
        Checkpoint(str(bad))


def test_checkpoint_integers(tmp_path):
    head = json.dumps({"t": {"dtype": "I32", "shape": [2, 2],
                             "data_offsets": [0, 16]}}).encode()
    f = tmp_path / "i.safetensors"
    f.write_bytes(struct.pack("<Q", len(head)) + head
                  + struct.pack("<4i", 1, -2, 3, 4))
    assert Checkpoint(str(f)).get("t").tolist() == [[1, -2], [3, 4]]


def test_registry_by_folder(tmp_path):
    cfg = CONFIGS["tiles"]
    folder = write_checkpoint(str(tmp_path / "m"), cfg,
                              random_weights(cfg, RANKS["tiles"]))
    got = get_config(folder + "#3")
    assert isinstance(got, KoridraConfig) and got.hidden == cfg["width"]
    assert [s.kind for s in got.layers] == [e["type"] for e in cfg["layers"]]
    assert [s.ff for s in got.layers] == [104, None, 64]
    assert got.layers[0].attn.chunk == 37 and got.needs_state
    model = build_model(folder, torch.device("cpu"))
    assert isinstance(model, KoridraModel) and model.embed.dtype \
        == torch.bfloat16
    (tmp_path / "x").mkdir()
    (tmp_path / "x" / "config.json").write_text('{"architecture": "None"}')
    with pytest.raises(KeyError):
        get_config(str(tmp_path / "x"))


def _broken(change):
    cfg = json.loads(json.dumps(CONFIGS["tiles"]))
    change(cfg["layers"])
    return cfg


@pytest.mark.parametrize("change", [
    lambda layers: layers[1].update(type="other"),
    lambda layers: layers[0]["mlp"].update(kind="sparse"),
    lambda layers: layers[1]["mixer"]["decay"].pop(),
    lambda layers: layers[0]["mixer"]["left"].update(vdim=8),
    lambda layers: layers[0]["mixer"]["left"].update(kv_heads=4)])
def test_config_that_is_not_the_design_is_refused(change):
    with pytest.raises(ValueError):
        KoridraConfig.from_dict(_broken(change))


def test_wrong_shape_is_refused(tmp_path):
    cfg = CONFIGS["odd"]
    w = random_weights(cfg, RANKS["odd"])
    w["l0.mix.v"] = w["l0.mix.v"][:-1]
    folder = write_checkpoint(str(tmp_path / "m"), cfg, w)
    with pytest.raises(ValueError):
        build_model(folder, torch.device("cpu"))


def test_preset_runs_and_sizes_add_up():
    cfg = get_config("koridra-tiny#0")
    model = build_model("koridra-tiny#0", torch.device("cpu"))
    again = build_model("koridra-tiny#0", torch.device("cpu"))
    other = build_model("koridra-tiny#1", torch.device("cpu"))
    assert torch.equal(model.head, again.head)
    assert not torch.equal(model.head, other.head)
    kv = model.new_kv_cache(3, 16, state_slots=2)
    assert kv.bytes() == 3 * 16 * cfg.kv_bytes_per_token() \
        + 3 * cfg.state_bytes_per_sequence()
    assert get_config("koridra-8b").param_count() > 6e9


def test_no_tensor_parallel_shards():
    from quoracle_amd.parallel.tp import TPContext
    with pytest.raises(NotImplementedError):
        build_model("koridra-tiny", torch.device("cpu"), tp=TPContext(0, 2))
