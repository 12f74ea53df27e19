"""The Kakirax design without a GPU: its configuration, and the plain restatement that the GPU tests compare with, one mechanism
at a time."""
import ctypes as C
import json
import os

import numpy as np
import pytest

from kakirax_cases import cases


@pytest.fixture(scope="module")
def ko():
    from oracle import kakirax_oracle
    return kakirax_oracle


def folder_config(fh, path, config):
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    c = fh.Config()
    fh.check(fh.lib().forge_hip_folder_config(str(path).encode(), C.byref(c)))
    return c


def test_sizes_come_from_the_configuration(fh, tmp_path):
    for name, (cfg, _) in cases(fh).items():
        c = folder_config(fh, tmp_path, cfg)
        first = next((l for l in cfg["layers"] if l["type"] == "attention"), cfg["layers"][0])["mixer"]
        assert (c.hidden, c.vocab, c.layers) == (cfg["width"], cfg["vocab"], len(cfg["layers"])), name
        assert (c.heads, c.kv_heads, c.head_dim) == (first["heads"], first.get("kv_heads", first["heads"]), first["dim"])
        assert c.inter == max((layer["mlp"] or {"ff": 0})["ff"] for layer in cfg["layers"])
        assert c.rms_eps == np.float32(cfg["norm"]["eps"]) and c.rope_theta == np.float32(first.get("rot", {"base": 0})["base"])


def test_logits_may_go_uncapped_and_null_means_absent(fh, tmp_path):
    cfg = json.loads(json.dumps(cases(fh)["uneven"][0]))
    cfg["layers"][3]["mixer"]["rot"]["scaling"] = None
    cfg["layers"][0]["weights_of"] = None
    folder_config(fh, tmp_path, cfg)
    cfg["logit_softcap"] = None
    folder_config(fh, tmp_path, cfg)
    del cfg["logit_softcap"]
    folder_config(fh, tmp_path, cfg)


def test_configurations_that_make_no_sense_are_refused(fh, tmp_path):
    def broken(change, message):
        cfg = json.loads(json.dumps(cases(fh)["uneven"][0]))
        change(cfg)
        with pytest.raises(fh.ForgeHipError, match=message) as e:
            folder_config(fh, tmp_path, cfg)
        assert e.value.code == fh.ERR_INVALID

    L = lambda c, i: c["layers"][i]
    broken(lambda c: c.update(logit_softcap=0), "logit_softcap")
    broken(lambda c: c.update(vocab=-1), "vocab")
    broken(lambda c: L(c, 0).update(type="latent_attention"), r"layers\[0\].type")
    broken(lambda c: L(c, 0)["mixer"].update(tau=0), r"layers\[0\].mixer.tau")
    broken(lambda c: L(c, 0)["mixer"].pop("vdim"), r"layers\[0\].mixer.vdim")
    broken(lambda c: L(c, 1)["mixer"].update(kv_heads=4), r"layers\[1\].mixer.kv_heads")
    broken(lambda c: L(c, 1)["mixer"]["rot"].update(dims=22), "rot")
    broken(lambda c: L(c, 1)["mixer"]["rot"].update(dims=5), "rot")
    broken(lambda c: L(c, 1)["mixer"]["rot"].update(scaling=3), "scaling")
    broken(lambda c: L(c, 1)["mixer"]["rot"]["scaling"].pop("original"), "scaling.original")
    broken(lambda c: L(c, 1)["mixer"]["rot"]["scaling"].update(factor=0), "scaling")
    broken(lambda c: L(c, 2)["mlp"].update(ff=0), "mlp.ff")
    broken(lambda c: L(c, 4).update(weights_of=7), r"layers\[4\].weights_of")
    broken(lambda c: L(c, 4).update(weights_of=1), r"layers\[4\].weights_of")
    broken(lambda c: L(c, 6)["mlp"].update(ff=129), r"layers\[6\].weights_of")
    broken(lambda c: (L(c, 0).update(weights_of=4)), "circle")


# ---- the plain restatement ------------------------------------------------------------------------------------------------------

def test_layer_norm(ko):
    x = np.array([[1.0, 2.0, 3.0, 6.0]])
    y = ko.layer_norm(x, np.array([1.0, 1.0, 2.0, 1.0]), np.array([0.0, 0.5, 0.0, 0.0]), 0.5)
    assert np.allclose(y, np.array([[-2.0, -1.0, 0.0, 3.0]]) / 2.0 * [1, 1, 2, 1] + [0, 0.5, 0, 0])       # variance 3.5, + 0.5: root 2
    assert np.allclose(ko.layer_norm(x + 100.0, np.ones(4), np.zeros(4), 0.1), ko.layer_norm(x, np.ones(4), np.zeros(4), 0.1))


def test_stretched_frequencies(ko):
    plain = ko.frequencies(64, 10000.0, None)
    assert np.allclose(plain, 10000.0 ** (-np.arange(32) / 32))
    sc = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 256}
    f, length = ko.frequencies(64, 10000.0, sc), 2 * np.pi / plain
    short, long = length < 64, length > 256
    assert short.any() and long.any() and (~short & ~long).any()
    assert np.array_equal(f[short], plain[short]) and np.allclose(f[long], plain[long] / 4)
    mid = f[~short & ~long] / plain[~short & ~long]
    assert np.all((mid > 0.25) & (mid < 1.0)) and np.all(np.diff(mid) < 0)
    # the blend meets both ends
    ends = [ko.frequencies(2, 1.0, dict(sc, original=o))[0] for o in (2 * np.pi * 1.0000001, 2 * np.pi * 3.9999999)]
    assert np.allclose(ends, [0.25, 1.0], atol=1e-6)


def test_rotation_depends_on_distance_only_and_leaves_the_rest(ko):
    rng = np.random.default_rng(0)
    a, b = rng.standard_normal((2, 1, 10))
    freq = ko.frequencies(8, 50.0, None)
    turn = lambda x, p: ko.rotate_half(x, np.array([p]), 8, freq)
    score = lambda p, q: (turn(a, p) @ turn(b, q).T).item()
    assert np.isclose(score(5, 2), score(105, 102)) and not np.isclose(score(5, 2), score(5, 3))
    assert np.array_equal(turn(a, 7)[:, 8:], a[:, 8:])
    e = np.zeros((1, 8))
    e[0, 1] = 1.0
    r = turn(e, 3)
    assert np.allclose(r[0, [1, 5]], [np.cos(3 * freq[1]), np.sin(3 * freq[1])]) and np.count_nonzero(r) == 2


def test_activations(ko):
    z = np.array([-40.0, -1.0, 0.0, 1.0, 40.0])
    assert np.allclose(ko.sigmoid(z), 1 / (1 + np.exp(-z))) and np.allclose(ko.log_sigmoid(z), -np.log1p(np.exp(-z)))
    assert np.allclose(ko.gelu_tanh(z), [0, -0.158808, 0, 0.841192, 40], atol=1e-6)
    assert np.allclose(ko.softcap(np.array([0.01, 1e6, -1e6]), 5.0), [0.01, 5, -5], atol=1e-5)


def test_the_recurrence_is_a_sum_over_earlier_tokens(ko):
    rng = np.random.default_rng(1)
    T, H, d, dv = 7, 2, 3, 5
    q, k, v, a = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, d)), rng.standard_normal((T, H, dv)), rng.uniform(0.1, 1, (T, H, d))
    o = ko.gated_state(q, k, v, a)
    for t in range(T):
        want = sum((q[t] * k[j] * np.prod(a[j + 1:t + 1], axis=0)).sum(-1)[:, None] * v[j] for j in range(t + 1))
        assert np.allclose(o[t], want)


def test_decay_is_a_root_of_the_sigmoid(ko):
    p = {"a1": np.array([[1.0, 0.0]]), "a2": np.array([[2.0], [0.0]]), "a2.b": np.array([0.0, -3.0])}
    a = ko.decays(np.array([[1.5, 9.0]]), p, {"tau": 4.0, "heads": 1, "dim": 2})
    assert a.shape == (1, 1, 2) and np.allclose(a[0, 0], [(1 / (1 + np.exp(-3.0))) ** 0.25, (1 / (1 + np.exp(3.0))) ** 0.25])


def test_heads_share_keys_in_order(ko):
    """Query heads 2 g and 2 g + 1 attend with key / value head g: values told apart by their head."""
    p = {"q": np.zeros((12, 4)), "k": np.zeros((6, 4)), "v": np.outer([1.0, 2.0, 3.0], [1, 0, 0, 0]), "g": np.zeros((6, 4)), "o": np.eye(6),
         "q.norm": np.ones(2), "k.norm": np.ones(2)}
    mix = {"heads": 6, "kv_heads": 3, "dim": 2, "vdim": 1, "scale": 1.0, "rot": {"base": 10.0, "dims": 2}}
    out = ko.attention(np.ones((3, 4)), p, mix, 1e-5)
    assert np.allclose(out, 0.5 * np.array([1, 1, 2, 2, 3, 3]))


def test_a_position_sees_nothing_later(fh, ko):
    cfg, rank = cases(fh)["uneven"]
    o = ko.Oracle(cfg, {k: fh.synth.from_bf16(v) for k, v in fh.synth.folder_tensors(cfg, 1, fh.synth.kakirax_shapes(cfg, rank)).items()})
    ids = np.random.default_rng(2).integers(0, cfg["vocab"], 20)
    base = o.forward(ids)[0]
    assert np.abs(base).max() <= cfg["logit_softcap"]
    for at in (0, 7, 19):
        other = ids.copy()
        other[at] = (other[at] + 1) % cfg["vocab"]
        assert (np.abs(o.forward(other)[0] - base).max(axis=1) > 1e-12).nonzero()[0].tolist() == list(range(at, 20))
