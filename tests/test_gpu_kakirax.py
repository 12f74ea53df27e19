"""The Kakirax network on the GPU, through the model handle, against the plain restatement in oracle/kakirax_oracle.py (64-bit)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from folder_model import DTYPES, LIMIT, ROOT, Case, check, decode_all, replay, row_errors
from kakirax_cases import cases

pytestmark = pytest.mark.gpu

NAMES = ["uneven", "many_heads", "wide", "middle", "ones", "attention_only", "linear_only"]


@pytest.fixture(scope="module")
def ko():
    from oracle import kakirax_oracle
    return kakirax_oracle


@pytest.fixture(scope="module")
def get(fh, ko, torch_gpu, tmp_path_factory):
    made, known = {}, cases(fh)

    def case(name):
        if name not in made:
            print("case", name, flush=True)
            cfg, rank = known[name]
            made[name] = Case(fh, ko, tmp_path_factory.mktemp(name), cfg, fh.synth.folder_tensors(cfg, 5, fh.synth.kakirax_shapes(cfg, rank)))
        return made[name]
    return case


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt(get, name, dtype):
    c = get(name)
    ids = c.ids(200)
    want, runs = c.oracle.forward(ids)
    m = c.model(dtype=dtype)
    assert m.config["hidden"] == c.cfg["width"] and m.decode_launches > 0
    check(m.prefill_logits(ids, np.arange(ids.size)), want, dtype)
    assert m.pos == ids.size
    m.reset()
    res = m.prefill_residuals(ids)
    assert res.shape == runs.shape and m.pos == 0
    for i in range(len(runs)):
        check(res[i], runs[i], dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_token_by_token(get, name, dtype):
    c = get(name)
    ids = c.ids(150, seed=10)
    want = c.oracle.forward(ids)[0]
    m = c.model(dtype=dtype)
    check(decode_all(m, ids), want, dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["uneven", "middle", "linear_only"])
def test_portions(get, name, dtype):
    """The prompt cut in portions of changing size, single tokens among them (one row of a prompt runs the decode kernels)."""
    c = get(name)
    ids = c.ids(230, seed=11)
    want = c.oracle.forward(ids)[0]
    m = c.model(dtype=dtype)
    for sizes in ([2], [3, 1, 2], [15, 17, 16], [64], [65, 63], [7, 100, 2, 33, 1, 1, 40, 47], [229, 1], [1, 229]):
        m.reset()
        at = k = 0
        while at < ids.size:
            n = min(sizes[k % len(sizes)], ids.size - at)
            check(m.prefill_logits(ids[at:at + n], np.arange(n)), want[at:at + n], dtype, np.sqrt((want ** 2).mean()))
            at, k = at + n, k + 1
        assert m.pos == ids.size
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["uneven", "many_heads", "linear_only"])
def test_prompts_of_every_length_around_the_tiles(get, name, dtype):
    """A prompt that ends just before, on and just behind a piece (16), a chunk (64) or a query tile (128), then decoded on."""
    c = get(name)
    ids = c.ids(200, seed=12)
    want = c.oracle.forward(ids)[0]
    m = c.model(dtype=dtype)
    for n in (1, 2, 3, 15, 16, 17, 31, 32, 33, 47, 48, 49, 63, 64, 65, 79, 80, 127, 128, 129, 191, 192, 193):
        m.reset()
        scale = np.sqrt((want ** 2).mean())
        check(m.prefill_logits(ids[:n], np.arange(n)[-64:]), want[:n][-64:], dtype, scale)
        check(decode_all(m, ids[n:n + 3]), want[n:n + 3], dtype, scale)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_requests_one_after_the_other(get, dtype):
    """What an earlier, longer request left in the cache, in the states and in the scratch areas does not show: the bits of a fresh
    model, whether a request begins with a prompt or with a decoded token."""
    c = get("uneven")
    requests = [c.ids(n, seed=20 + n) for n in (190, 5, 77, 1, 130)]
    used = c.model(dtype=dtype)
    for ids in requests:
        fresh = c.model(dtype=dtype)
        for cut in {0, max(1, ids.size - 6)}:
            got = []
            for m in (used, fresh):
                m.reset()
                got.append(([m.prefill_logits(ids[:cut], np.arange(cut))] if cut else []) + [m.forward(int(t)) for t in ids[cut:cut + 9]])
            for a, b in zip(*got):
                assert np.array_equal(a.view(np.uint32), b.view(np.uint32))
        fresh.close()
    used.close()


def test_the_captured_step_equals_the_eager_one(get, monkeypatch):
    """The decode step replayed as a graph, with prompts and eager steps between the replays, against a model without graphs."""
    c = get("uneven")
    ids = c.ids(60, seed=31)
    a = c.model()
    monkeypatch.setenv("FORGE_HIP_GRAPH", "0")
    b = c.model()
    for m in (a, b):
        m.forward_prefill_batch(ids[:20])
    for i in range(20, 60):
        if i % 7 == 0:
            x, y = (m.prefill_logits(ids[i:i + 1], [0])[0] for m in (a, b))
        else:
            x, y = (m.forward(int(ids[i])) for m in (a, b))
        assert np.array_equal(x.view(np.uint32), y.view(np.uint32)), i
    a.close()
    b.close()


def test_shared_weights_equal_copied_ones(get, fh, ko, tmp_path):
    """A layer that names another layer's tensors gives the bits of one that has copies of them, each with a cache of its own."""
    c = get("uneven")
    cfg, t = copy.deepcopy(c.cfg), dict(c.tensors)
    for i, layer in enumerate(cfg["layers"]):
        of = layer.pop("weights_of", None)
        if of is not None:
            t.update({"l%d." % i + k[len("l%d." % of):]: v for k, v in c.tensors.items() if k.startswith("l%d." % of)})
    d = Case(fh, ko, tmp_path, cfg, t)
    ids = c.ids(90, seed=13)
    a, b = c.model(), d.model()
    for m in (a, b):
        assert m.pos == 0
    x, y = (np.concatenate([m.prefill_logits(ids[:80], np.arange(80)), decode_all(m, ids[80:])]) for m in (a, b))
    assert np.array_equal(x.view(np.uint32), y.view(np.uint32))
    a.close()
    b.close()


# ---- inputs under which one key stands out ---------------------------------------------------------------------------------------

def told_apart(fh, ko, path, layer, rng, key_of, query_of, decay_bias=None):
    """One layer of one mixer whose input vectors are the rows of a Hadamard matrix (entries +-1, each with mean 0, orthogonal): a
    projection can give every token any query, key and value.  key_of, query_of: [63][dim], the same for all heads."""
    hadamard = np.ones((1, 1))
    for _ in range(6):
        hadamard = np.block([[hadamard, hadamard], [hadamard, -hadamard]])
    rows = hadamard[1:]
    cfg = fh.synth.kakirax_config(64, 63, [layer], cap=40.0)
    t = fh.synth.folder_tensors(cfg, 3)
    t["embed"] = fh.synth.to_bf16(rows)
    for n, v in (("l0.norm1", np.ones(64)), ("l0.norm1.b", np.zeros(64))):
        t[n] = fh.synth.to_bf16(v)
    mix = layer["mixer"]
    maps = lambda table, heads: fh.synth.to_bf16(np.concatenate([table] * heads, axis=1).T @ rows / 64)
    t["l0.mix.q"] = maps(query_of, mix["heads"])
    t["l0.mix.k"] = maps(key_of, mix.get("kv_heads", mix["heads"]))
    t["l0.mix.v"] = fh.synth.to_bf16(rng.standard_normal((mix.get("kv_heads", mix["heads"]) * mix["vdim"], 63)) @ rows / 64)
    if decay_bias is not None:
        t["l0.mix.a2"] = np.zeros_like(t["l0.mix.a2"])
        t["l0.mix.a2.b"] = fh.synth.to_bf16(np.full(t["l0.mix.a2.b"].shape, decay_bias))
    return Case(fh, ko, path, cfg, t)


QUERY, KEY = 0, 1
FILL = np.arange(2, 63)


def needle_attention(fh, ko, path, kv_heads):
    """Scores that hardly depend on the places (one slow pair turns): the key token's is far above all others."""
    rng = np.random.default_rng(6)
    d = 24
    k = rng.standard_normal((63, d))
    q = rng.standard_normal((63, d))
    q[QUERY] = 4.0 * np.sign(rng.standard_normal(d))
    k[KEY] = q[QUERY]
    k[FILL] -= 0.8 * np.sign(q[QUERY])
    k[QUERY] = k[FILL[0]]
    k[:, [0, 1]] = q[:, [0, 1]] = 0.01                    # the pair that turns
    return told_apart(fh, ko, path, fh.synth.kakirax_attention(4, kv_heads, d, 20, None, scale=0.7, rot_dims=2), rng, k, q)


def needle_linear(fh, ko, path):
    """Decays of nearly 1: what the key token left in the state is there unweakened, and far above the rest."""
    rng = np.random.default_rng(7)
    d = 12
    k = 0.01 * rng.standard_normal((63, d))
    q = rng.standard_normal((63, d))
    k[KEY] = 8.0 * q[QUERY]
    return told_apart(fh, ko, path, fh.synth.kakirax_gla(3, d, 20, None, tau=2.0), rng, k, q, decay_bias=30.0)


def stands_out(c, ids, at, want, dtype):
    lost = ids.copy()
    lost[at] = FILL[3]
    return row_errors(c.oracle.forward(lost)[0][-1], want[-1]).max() > 5 * LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "attention_one_kv_head", "linear"])
def test_far_key(fh, ko, torch_gpu, tmp_path, kind, dtype):
    """One key among hundreds: at the ends, and at the borders of the kernels' pieces, chunks, tiles and parts; the query in a
    prompt, in a later portion, and decoded."""
    c = needle_linear(fh, ko, tmp_path) if kind == "linear" else needle_attention(fh, ko, tmp_path, 2 if kind == "attention" else 1)
    rng = np.random.default_rng(2)
    m = c.model(max_seq=1024, dtype=dtype)
    for n, places in ((900, (0, 1, 15, 16, 63, 64, 447, 448, 512, 831, 897, 898)), (130, (0, 16, 64, 127, 128)), (65, (0, 47, 48, 63)), (3, (0, 1))):
        for at in places:
            ids = FILL[rng.integers(0, FILL.size, n)]
            ids[-1], ids[at] = QUERY, KEY
            want = c.oracle.forward(ids)[0]
            assert stands_out(c, ids, at, want, dtype)
            m.reset()
            check(m.forward_prefill(ids), want[-1], dtype)
            m.reset()
            m.forward_prefill_batch(ids[:-1])
            check(m.forward(QUERY), want[-1], dtype)
            cut = max(1, min(at + 1, n - 2))              # the first portion ends with the key
            m.reset()
            m.forward_prefill_batch(ids[:cut])
            check(m.prefill_logits(ids[cut:], [n - cut - 1])[0], want[-1], dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("first", [1, 63, 64, 65, 130])
def test_key_that_passes_over_decoded_tokens(fh, ko, torch_gpu, tmp_path, first, dtype):
    """The key is decoded, then fillers, then the query: every place of a tile is written by a decode step."""
    c = needle_linear(fh, ko, tmp_path / "linear")
    a = needle_attention(fh, ko, tmp_path / "attention", 2)
    rng = np.random.default_rng(3)
    for case in (c, a):
        m = case.model(dtype=dtype)
        ids = FILL[rng.integers(0, FILL.size, first + 75)]
        ids[first], ids[first + 64], ids[-1] = KEY, QUERY, QUERY
        want = case.oracle.forward(ids)[0]
        assert stands_out(case, ids, first, want, dtype)
        m.forward_prefill_batch(ids[:first])
        check(decode_all(m, ids[first:]), want[first:], dtype, np.sqrt((want ** 2).mean()))
        m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bias,tau", [(-90.0, 1.0), (-6.0, 1.0), (-1.0, 16.0), (3.0, 0.5), (40.0, 1.0)])
def test_decays_of_every_strength(fh, ko, torch_gpu, tmp_path, bias, tau, dtype):
    """From a state that forgets everything at once (products of decays underflow) to one that forgets nothing."""
    cfg = fh.synth.kakirax_config(48, 70, [fh.synth.kakirax_gla(2, 40, 24, None, tau=tau)], embedding_scale=7.0)
    t = fh.synth.folder_tensors(cfg, 4)
    spread = np.random.default_rng(1).uniform(0.2, 1.0, 80) * bias
    t["l0.mix.a2.b"] = fh.synth.to_bf16(spread)
    c = Case(fh, ko, tmp_path, cfg, t)
    ids = c.ids(180, seed=14)
    want = c.oracle.forward(ids)[0]
    m = c.model(dtype=dtype)
    check(m.prefill_logits(ids, np.arange(ids.size)), want, dtype)
    m.reset()
    m.forward_prefill_batch(ids[:70])
    check(decode_all(m, ids[70:130]), want[70:130], dtype, np.sqrt((want ** 2).mean()))
    check(m.prefill_logits(ids[130:], np.arange(50)), want[130:], dtype, np.sqrt((want ** 2).mean()))
    m.close()


def test_stretched_rotation(fh, ko, torch_gpu, tmp_path):
    """Waves kept, blended and slowed, far enough into a sequence that each rule shows."""
    lay = fh.synth.kakirax_attention(2, 1, 32, 16, None, base=300.0, scaling=(6.0, 1.0, 4.0, 100), scale=1.0)
    cfg = fh.synth.kakirax_config(48, 70, [lay], embedding_scale=7.0)
    c = Case(fh, ko, tmp_path, cfg)
    ids = c.ids(600, seed=15)
    want = c.oracle.forward(ids)[0]
    for change in ({"factor": 1.0}, {"high": 1.0001}, {"low": 3.9}):
        other = copy.deepcopy(cfg)
        other["layers"][0]["mixer"]["rot"]["scaling"].update(change)
        assert row_errors(ko.Oracle(other, c.oracle.t).forward(ids)[0], want).max() > 5 * LIMIT["float32"], change
    m = c.model(max_seq=600)
    check(m.prefill_logits(ids[:560], np.arange(500, 560)), want[500:560], "float32")
    check(decode_all(m, ids[560:]), want[560:], "float32")
    m.close()


def test_long_decoding(get, fh):
    """Up to the last position of the cache."""
    c = get("uneven")
    ids = c.ids(512, seed=41)
    want = c.oracle.forward(ids)[0]
    m = c.model(max_seq=512)
    m.forward_prefill_batch(ids[:30])
    check(decode_all(m, ids[30:]), want[30:], "float32")
    with pytest.raises(fh.ForgeHipError) as e:
        m.forward(0)
    assert e.value.code == fh.ERR_POSITION
    m.reset()
    with pytest.raises(fh.ForgeHipError) as e:
        m.forward_prefill_batch(np.zeros(513, np.uint32))
    assert e.value.code == fh.ERR_POSITION
    check(m.forward_prefill(ids[:40]), want[39], "float32")              # a refused call leaves the model usable
    m.close()


def test_prompt_past_one_chunk(fh, ko, torch_gpu, tmp_path):
    """A prompt longer than the rows of scratch: the second chunk goes on from the first one's cache and states."""
    cfg = fh.synth.kakirax_config(40, 50, [fh.synth.kakirax_gla(2, 16, 16, 30, tau=200.0), fh.synth.kakirax_attention(2, 1, 16, 16, None), 0], embedding_scale=6.0)
    c = Case(fh, ko, tmp_path, cfg)
    ids = c.ids(4161, seed=51)
    want = c.oracle.forward(ids)[0]
    m = c.model(max_seq=4224)
    rows = np.r_[0, 2000, 4090:4160]
    check(m.prefill_logits(ids[:-1], rows), want[rows], "float32")
    check(m.forward(int(ids[-1])), want[-1], "float32")
    m.close()


# ---- one mechanism at a time ------------------------------------------------------------------------------------------------------

def test_mechanisms_alone(fh, ko, torch_gpu, tmp_path):
    att = fh.synth.kakirax_attention(4, 2, 18, 10, 25, base=90.0, rot_dims=14, scaling=(3.0, 1.0, 5.0, 60), scale=0.5)
    gla = fh.synth.kakirax_gla(3, 12, 20, 25, tau=5.0)
    rng = np.random.default_rng(5)
    ids = rng.integers(0, 60, 90)
    for kind, lay in (("attention", att), ("gla", gla)):
        cfg = fh.synth.kakirax_config(50, 60, [lay], embedding_scale=2.5, eps=0.02, cap=3.0)
        base = fh.synth.folder_tensors(cfg, 8)
        f = {k: fh.synth.from_bf16(v).astype(np.float64) for k, v in base.items()}
        norm = lambda x, n: ko.layer_norm(x, f[n], f[n + ".b"], 0.02)
        part = lambda prefix: {k[len(prefix):]: v for k, v in f.items() if k.startswith(prefix)}
        x0 = f["embed"][ids] * 2.5

        def run(name, *silent):
            t = {k: np.zeros_like(v) if k in silent else v for k, v in base.items()}
            c = Case(fh, ko, tmp_path / (kind + name), cfg, t)
            m = c.model()
            out = m.prefill_residuals(ids)[0], m.prefill_logits(ids, np.arange(ids.size))
            m.close()
            return out

        x, logits = run("nothing", "l0.mix.o", "l0.mlp.down")
        check(x, x0, "float32")                                                  # the embedding and its scale
        want = ko.softcap(norm(x0, "final.norm") @ f["embed"].T, 3.0)            # final norm, table as output matrix, cap
        check(logits, want, "float32")
        a = ko.MIXERS[kind](norm(x0, "l0.norm1"), part("l0.mix."), lay["mixer"], 0.02)
        check(run("mixer", "l0.mlp.down")[0] - x0, a, "float32")
        b = ko.gated_ff(norm(x0, "l0.norm2"), part("l0.mlp."))
        check(run("ff", "l0.mix.o")[0] - x0, b, "float32")


def test_the_cap_bends_large_logits_only(fh, ko, torch_gpu, tmp_path):
    cfg = fh.synth.kakirax_config(64, 63, [fh.synth.kakirax_gla(1, 8, 8, None)], embedding_scale=1.0)
    t = fh.synth.folder_tensors(cfg, 2)
    for cap in (0.5, 1000.0, None):
        c = Case(fh, ko, tmp_path / str(cap), dict(cfg, logit_softcap=cap or 1e30), t)
        want = c.oracle.forward(c.ids(20))[0]
        if cap is None:
            fh.synth.write_model_folder(c.path, dict(cfg, logit_softcap=None), t)
        m = c.model()
        check(m.prefill_logits(c.ids(20), np.arange(20)), want, "float32")
        m.reset()
        check(decode_all(m, c.ids(20)), want, "float32")
        m.close()


# ---- generation, loading, replay --------------------------------------------------------------------------------------------------

def test_greedy_generation(get):
    """The framework's generation loop (prompt, then forward_greedy with the argmax on the device) against the oracle's."""
    c = get("uneven")
    prompt = c.ids(40, seed=61)
    want = c.oracle.greedy(prompt, 24)
    m = c.model()
    assert m.generate_greedy(prompt, 24) == want
    m.reset()
    assert m.generate(prompt, max_tokens=24, repeat_penalty=1.0) == want
    m.reset()
    m.set_repeat_penalty(1.0)
    sampled = m.generate(prompt, max_tokens=12, temperature=0.8, repeat_penalty=1.0, seed=77)
    m.reset()
    assert m.generate(prompt, max_tokens=12, temperature=0.8, repeat_penalty=1.0, seed=77) == sampled
    m.close()


def test_chat_server_serves_the_model(get, fh):
    c = get("attention_only")

    class Ids:
        """A tokenizer of one token per character."""
        def encode(self, text, add_special_tokens):
            return [ord(ch) % 150 for ch in text]

        def decode(self, ids, skip_special_tokens):
            return "<%d>" % ids[0]

    m = c.model()
    body = json.dumps({"messages": [{"role": "user", "content": "hello"}], "max_tokens": 6}).encode()
    server = fh.serve.ChatServer(m, Ids())
    prompt = Ids().encode(fh.serve.format_chat_messages([{"role": "user", "content": "hello"}]), True)
    want = c.oracle.greedy(prompt, 6)
    want = want[:want.index(2)] if 2 in want else want
    for _ in range(2):                                   # the second request takes the first one's place
        status, _, answer = server.handle("POST", "/v1/chat/completions", body)
        assert status == 200 and json.loads(answer)["choices"][0]["message"]["content"] == "".join("<%d>" % t for t in want)
    m.close()


def test_profiles_count_every_launch(get):
    c = get("uneven")
    m = c.model()
    m.forward_prefill_batch(c.ids(20))
    prof = m.forward_profile(3)
    assert sum(n for _, n in prof.values()) == m.decode_launches and m.pos == 21
    assert prof["attention"][0] > 0 and prof["lm_head_matmul"][1] == 1
    m.reset()
    pre = m.prefill_profile(c.ids(20))
    assert pre["gate_up_matmul"][1] == 4 and pre["o_matmul"][1] == 7               # of seven layers four have a feed-forward
    m.close()


def test_refusals(get, fh, tmp_path):
    c = get("middle")
    m = c.model()
    with pytest.raises(fh.ForgeHipError, match="flat cache"):
        m.set_kv_pages(64, np.arange(4))
    with pytest.raises(fh.ForgeHipError):
        m.forward_prefill_batch([c.cfg["vocab"]])
    m.close()
    shapes = fh.synth.kakirax_shapes(c.cfg, 33)
    for name, change in (("a1", lambda t: t.pop("l0.mix.a1")), ("a2", lambda t: t.update({"l0.mix.a2": t["l0.mix.a2"][:, :-1]})),
                         ("norm", lambda t: t.pop("l2.mix.q.norm")), ("bias", lambda t: t.pop("final.norm.b"))):
        bad = dict(c.tensors)
        change(bad)
        fh.synth.write_model_folder(str(tmp_path / name), c.cfg, bad)
        with pytest.raises(fh.ForgeHipError, match="tensor"):
            fh.HipModel.from_folder(str(tmp_path / name), 64)
    assert len(shapes) == len(c.tensors)
    for name, layer, size in (("dim", 2, {"dim": 258}), ("vdim", 0, {"vdim": 257})):
        big = copy.deepcopy(c.cfg)
        big["layers"][layer]["mixer"].update(size)
        fh.synth.write_model_folder(str(tmp_path / ("big" + name)), big, fh.synth.folder_tensors(big, 1))
        with pytest.raises(fh.ForgeHipError, match="256"):
            fh.HipModel.from_folder(str(tmp_path / ("big" + name)), 64)


def test_command_line(get):
    c = get("uneven")
    prompt = c.ids(12, seed=62)
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), c.path, "--ids", ",".join(map(str, prompt)), "--max-tokens", "9",
                        "--repeat-penalty", "1", "--dtype", "float32"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split()[-1].split(",")] == c.oracle.greedy(prompt, 9)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(get, tmp_path, dtype):
    """bin/trace_run on a small trace: requests one after the other, prompt portions and single tokens."""
    c = get("uneven")
    replay(c, {"a": c.ids(70, seed=71), "b": c.ids(33, seed=72), "c": c.ids(1, seed=73)}, (40, 1, 2, 1, 1000), dtype, tmp_path)
