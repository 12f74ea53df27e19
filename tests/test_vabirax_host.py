"""Model folders without a GPU: the configuration reader and its registry, the safetensors reader, and the plain restatement of
the design that the GPU tests compare with."""
import json
import os

import numpy as np
import pytest

from vabirax_cases import cases


@pytest.fixture(scope="module")
def vo():
    from oracle import vabirax_oracle
    return vabirax_oracle


def folder_config(fh, path):
    import ctypes as C
    c = fh.Config()
    fh.check(fh.lib().forge_hip_folder_config(str(path).encode(), C.byref(c)))
    return c


def write(path, config):
    with open(os.path.join(path, "config.json"), "w") as f:
        f.write(config if isinstance(config, str) else json.dumps(config))


def test_sizes_come_from_the_configuration(fh, tmp_path):
    for name, cfg in cases(fh).items():
        write(tmp_path, cfg)
        c = folder_config(fh, tmp_path)
        m = cfg["layers"][0]["mixer"]
        assert (c.hidden, c.vocab, c.layers, c.heads) == (cfg["width"], cfg["vocab"], len(cfg["layers"]), m["heads"]), name
        assert c.head_dim == m["dim"] + m["rot_dim"] and c.sliding_window == m.get("mask", {}).get("size", 0)
        assert c.inter == max((layer["mlp"] or {"ff": 0})["ff"] for layer in cfg["layers"])
        assert c.rms_eps == np.float32(cfg["norm"]["eps"]) and c.rope_theta == np.float32(m["rot"]["base"])


def test_configurations_that_make_no_sense_are_refused(fh, tmp_path):
    def broken(change, message):
        cfg = json.loads(json.dumps(cases(fh)["uneven"]))
        change(cfg)
        write(tmp_path, cfg)
        with pytest.raises(fh.ForgeHipError, match=message) as e:
            folder_config(fh, tmp_path)
        assert e.value.code == fh.ERR_INVALID

    broken(lambda c: c.pop("architecture"), "architecture")
    broken(lambda c: c.update(architecture="Vabirax2"), "unknown architecture")
    broken(lambda c: c.update(width=0), "width")
    broken(lambda c: c.update(vocab=3.5), "vocab")
    broken(lambda c: c.update(layers=[]), "layers")
    broken(lambda c: c["layers"][1].update(type="attention"), r"layers\[1\].type")
    broken(lambda c: c["layers"][2]["mixer"].pop("kv_rank"), r"layers\[2\].mixer.kv_rank")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), "rot")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8), "rot")
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size")
    broken(lambda c: c["layers"][0]["mlp"].update(kind="routed"), "mlp.kind")
    broken(lambda c: c["loop"].update(stop=9), "loop")
    broken(lambda c: c["loop"].update(times=0), "loop.times")


@pytest.mark.parametrize("text", ["", "{", '{"architecture": "Vabirax",}', '{"a": 1} x', '{"a": tru}', '{"a": 1e}', '["\\u12"]', '"abc',
                                  '{"a" 1}', "[" * 100])
def test_broken_json_is_refused(fh, tmp_path, text):
    write(tmp_path, text)
    with pytest.raises(fh.ForgeHipError, match="JSON"):
        folder_config(fh, tmp_path)


def test_json_escapes_and_nesting(fh, tmp_path):
    cfg = cases(fh)["no_window"]
    text = json.dumps(dict(cfg, note={"s": 'a"\\/\b\f\n\r\té€\U0001F600', "l": [None, True, False, -1.5e-3, {}, []]}), indent=3)
    write(tmp_path, text.replace('"Vabirax"', '"\\u0056abirax"'))
    assert folder_config(fh, tmp_path).vocab == cfg["vocab"]


def test_missing_folder_and_broken_safetensors(fh, tmp_path):
    with pytest.raises(fh.ForgeHipError, match="config.json"):
        fh.HipModel.from_folder(str(tmp_path / "nowhere"))
    cfg = cases(fh)["ones"]
    st = tmp_path / "model.safetensors"

    def refused(data, message):
        write(tmp_path, cfg)
        st.write_bytes(data)
        with pytest.raises(fh.ForgeHipError, match=message):
            fh.HipModel.from_folder(str(tmp_path))

    def file(header, body=b""):
        h = json.dumps(header).encode()
        return len(h).to_bytes(8, "little") + h + body

    refused(b"1234", "too short")
    refused((1 << 40).to_bytes(8, "little") + b"{}", "longer than the file")
    refused(file([]), "not an object")
    refused(file({"embed": {"dtype": "BF16", "shape": [2]}}), "not described")
    refused(file({"embed": {"dtype": "F8_E4M3", "shape": [2], "data_offsets": [0, 2]}}, b"12"), "F8_E4M3")
    refused(file({"embed": {"dtype": "BF16", "shape": [2], "data_offsets": [0, 4]}}, b"12"), "does not lie in the file")
    refused(file({"embed": {"dtype": "BF16", "shape": [2], "data_offsets": [0, 2]}}, b"12"), "does not lie in the file")
    refused(file({"embed": {"dtype": "BF16", "shape": [4294967295, 4294967295, 4294967295], "data_offsets": [0, 2]}}, b"12"), "impossible shape")


def test_bfloat16_helpers(fh):
    x = np.array([0.0, -0.0, 1.0, 1.00390625, 1.01171875, 3.1415927, -1e-30, 65504.0], np.float32)
    back = fh.synth.from_bf16(fh.synth.to_bf16(x))
    assert np.all(np.abs(back - x) <= np.abs(x) * 2.0 ** -8)
    assert fh.synth.from_bf16(fh.synth.to_bf16(np.float32([1.00390625, 1.01171875]))).tolist() == [1.0, 1.015625]      # ties to even


# ---- the plain restatement ------------------------------------------------------------------------------------------------------

def test_window_counts_the_position_itself(vo):
    ok = vo.window_mask(6, 3)
    assert [row.nonzero()[0].tolist() for row in ok] == [[0], [0, 1], [0, 1, 2], [1, 2, 3], [2, 3, 4], [3, 4, 5]]
    assert np.array_equal(vo.window_mask(5, 1), np.eye(5, dtype=bool)) and np.array_equal(vo.window_mask(4, None), np.tri(4, dtype=bool))


def test_rotation_depends_on_distance_only_and_leaves_the_rest(vo):
    rng = np.random.default_rng(0)
    a, b = rng.standard_normal((2, 1, 10))
    score = lambda p, q: (vo.rotate_half(a, np.array([p]), 8, 100.0) @ vo.rotate_half(b, np.array([q]), 8, 100.0).T).item()
    assert np.isclose(score(5, 2), score(105, 102)) and not np.isclose(score(5, 2), score(5, 3))
    assert np.array_equal(vo.rotate_half(a, np.array([7]), 8, 100.0)[:, 8:], a[:, 8:])
    # pair (1, 5) of 8 turns by position * base^(-2/8)
    e = np.zeros((1, 8))
    e[0, 1] = 1.0
    r = vo.rotate_half(e, np.array([3]), 8, 16.0)
    assert np.allclose(r[0, [1, 5]], [np.cos(1.5), np.sin(1.5)]) and np.count_nonzero(r) == 2


def test_order_of_looped_layers(vo):
    base = {"layers": [None] * 5}
    assert vo.layer_order(base) == [(i, False) for i in range(5)]
    looped = dict(base, loop={"start": 1, "stop": 3, "times": 2})
    assert vo.layer_order(looped) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]
    assert vo.layer_order(dict(base, loop={"start": 0, "stop": 5, "times": 1})) == [(0, True)] + [(i, False) for i in range(1, 5)]


def test_norms(vo):
    x = np.array([[3.0, -4.0]])
    assert np.allclose(vo.rms(x, np.array([1.0, 2.0]), 0.0), [[3 / np.sqrt(12.5), -8 / np.sqrt(12.5)]])
    assert np.allclose(vo.dyn_tanh(x, 0.5, np.array([2.0, 1.0]), np.array([0.1, -0.1])), [[2 * np.tanh(1.5) + 0.1, np.tanh(-2.0) - 0.1]])


def test_a_position_sees_nothing_later_and_nothing_before_its_windows(fh, vo):
    cfg = fh.synth.vabirax_config(24, 30, [fh.synth.vabirax_layer(2, 8, 4, 8, 12, 16, 20, 4)] * 2)
    t = {k: fh.synth.from_bf16(v) for k, v in fh.synth.folder_tensors(cfg, 1).items()}
    o = vo.Oracle(cfg, t)
    ids = np.random.default_rng(2).integers(0, 30, 20)
    base = o.forward(ids)[0]
    for at in (0, 7, 13):
        other = ids.copy()
        other[at] = (other[at] + 1) % 30
        moved = np.abs(o.forward(other)[0] - base).max(axis=1) > 1e-9
        assert moved.nonzero()[0].tolist() == list(range(at, min(20, at + 7)))        # two layers of three steps back each
