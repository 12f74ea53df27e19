"""The Vabirax network on the GPU, through the model handle, against the plain restatement in oracle/vabirax_oracle.py (64-bit)."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from folder_model import DTYPES, LIMIT, Case, check, decode_all, replay
from vabirax_cases import cases

pytestmark = pytest.mark.gpu

NAMES = ["uneven", "many_heads", "wide_head", "large_rank", "ones", "no_window", "part_rotation"]


@pytest.fixture(scope="module")
def vo():
    from oracle import vabirax_oracle
    return vabirax_oracle


@pytest.fixture(scope="module")
def get(fh, vo, torch_gpu, tmp_path_factory):
    made, known = {}, cases(fh)

    def case(name):
        if name not in made:
            print("case", name, flush=True)
            made[name] = Case(fh, vo, tmp_path_factory.mktemp(name), known[name])
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
@pytest.mark.parametrize("name", ["uneven", "many_heads", "no_window"])
def test_portions(get, name, dtype):
    """The prompt cut in portions of changing size, single tokens among them (one row of a prompt runs the decode kernels)."""
    c = get(name)
    ids = c.ids(230, seed=11)
    want = c.oracle.forward(ids)[0]
    m = c.model(dtype=dtype)
    for sizes in ([2], [3, 1, 2], [64], [65, 63], [7, 100, 2, 33, 1, 1, 40, 47], [229, 1]):
        m.reset()
        at = k = 0
        while at < ids.size:
            n = min(sizes[k % len(sizes)], ids.size - at)
            check(m.prefill_logits(ids[at:at + n], np.arange(n)), want[at:at + n], dtype, np.sqrt((want ** 2).mean()))
            at, k = at + n, k + 1
        assert m.pos == ids.size
    m.close()


@pytest.mark.parametrize("name", ["uneven", "wide_head", "no_window"])
def test_first_tokens(get, name):
    c = get(name)
    ids = c.ids(4, seed=12)
    m = c.model()
    for n in (1, 2, 3, 4):
        want = c.oracle.forward(ids[:n])[0]
        m.reset()
        check(m.forward_prefill(ids[:n]), want[-1], "float32")
        m.reset()
        check(decode_all(m, ids[:n]), want, "float32")
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_requests_one_after_the_other(get, dtype):
    """What an earlier, longer request left in the cache and in the scratch areas does not show: the bits of a fresh model."""
    c = get("uneven")
    requests = [c.ids(n, seed=20 + n) for n in (190, 5, 77, 1, 130)]
    used = c.model(dtype=dtype)
    for ids in requests:
        fresh = c.model(dtype=dtype)
        cut = max(1, ids.size - 6)
        got = []
        for m in (used, fresh):
            m.reset()
            got.append([m.prefill_logits(ids[:cut], np.arange(cut))] + [m.forward(int(t)) for t in ids[cut:]])
        fresh.close()
        for a, b in zip(*got):
            assert np.array_equal(a.view(np.uint32), b.view(np.uint32))
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


def needle_case(fh, vo, path, window, seed=3):
    """One layer whose scores depend on the two tokens only (the queries' rotated part is zero), sharpened so that for a query
    token one key token takes nearly all the weight.  Returns the case, the query token, the key token and filler tokens with
    low scores."""
    cfg = fh.synth.vabirax_config(60, 80, [fh.synth.vabirax_layer(2, 24, 8, 20, 32, 40, None, window, scale=4.0)])
    t = fh.synth.folder_tensors(cfg, seed)
    uq = fh.synth.from_bf16(t["l0.mix.uq"]).reshape(2, 32, 32)
    uq[:, 24:] = 0.0
    uq[1] = uq[0]                                                         # both heads look for the same key
    uk = fh.synth.from_bf16(t["l0.mix.uk"]).reshape(2, 24, 40)
    uk[1] = uk[0]
    t["l0.mix.uq"], t["l0.mix.uk"] = fh.synth.to_bf16(uq).reshape(64, 32), fh.synth.to_bf16(uk).reshape(48, 40)
    c = Case(fh, vo, path, cfg, t)
    o = c.oracle
    p = o._part("l0.mix.")
    h = o.norm(o.t["embed"] * cfg["embedding"]["scale"], "l0.norm1")
    q = (vo.rms(h @ p["dq"].T, p["dq.norm"], 1e-5) @ p["uq"].T)[:, :24]
    k = vo.rms((h @ p["dkv"].T)[:, :40], p["dkv.norm"], 1e-5) @ p["uk"].T
    s = q @ k[:, :24].T * 4.0
    query, key = np.unravel_index((s - np.diag(s)[:, None]).argmax(), s.shape)
    fill = np.argsort(s[query])[:30]
    assert s[query, key] - max(s[query, fill].max(), s[query, query]) > np.log(2000.0)
    return c, int(query), int(key), fill


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [2, 31, 64, 65, 200])
def test_window_edges(fh, vo, torch_gpu, tmp_path, window, dtype):
    """A key that takes nearly all the weight, placed on the last visible position, one further away and one nearer, for queries
    around tile borders, in a prompt and decoded."""
    c, query, key, fill = needle_case(fh, vo, tmp_path, window)
    rng = np.random.default_rng(1)
    m = c.model(max_seq=512, dtype=dtype)
    for i in (window, 63, 64, 127, 128, 129, 191, 255, 300):
        rows = []
        for distance in (window - 1, window, window - 2):
            if distance > i or distance < 1:
                continue
            ids = fill[rng.integers(0, fill.size, i + 1)]
            ids[i], ids[i - distance] = query, key
            want = c.oracle.forward(ids)[0]
            m.reset()
            check(m.prefill_logits(ids, np.arange(i + 1)), want, dtype)
            m.reset()
            if i:
                m.forward_prefill_batch(ids[:i])
            check(m.forward(query), want[-1], dtype)
            # a window one off would be seen: compare with the same tokens under the shifted window
            off = json.loads(json.dumps(c.cfg))
            off["layers"][0]["mixer"]["mask"]["size"] = window + (1 if distance == window else -1)
            if distance != window - 2:
                wrong = vo.Oracle(off, c.oracle.t).forward(ids)[0][-1]
                rows.append(np.sqrt(((wrong - want[-1]) ** 2).mean()) / np.sqrt((want ** 2).mean()))
        assert all(r > 5 * LIMIT[dtype] for r in rows), rows
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key(fh, vo, torch_gpu, tmp_path, dtype):
    """One key among hundreds, without a mask: at the ends, at tile borders and where the decode attention's parts meet."""
    c, query, key, fill = needle_case(fh, vo, tmp_path, None)
    rng = np.random.default_rng(2)
    m = c.model(max_seq=1024, dtype=dtype)
    for n, places in ((900, (0, 1, 63, 64, 447, 448, 512, 831, 897)), (129, (0, 64, 127))):
        for at in places:
            ids = fill[rng.integers(0, fill.size, n)]
            ids[-1], ids[at] = query, key
            want = c.oracle.forward(ids)[0]
            m.reset()
            check(m.forward_prefill(ids), want[-1], dtype)
            m.reset()
            m.forward_prefill_batch(ids[:-1])
            check(m.forward(query), want[-1], dtype)
            lost = ids.copy()
            lost[at] = fill[0]
            without = c.oracle.forward(lost)[0][-1]
            assert np.sqrt(((without - want[-1]) ** 2).mean()) > 5 * LIMIT[dtype] * np.sqrt((want[-1] ** 2).mean())
    m.close()


def test_long_decoding(get, fh):
    """Far past the windows, up to the last position of the cache."""
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


def test_prompt_past_one_chunk(fh, vo, torch_gpu, tmp_path):
    """A prompt longer than the rows of scratch: the second chunk's first windows reach back into the first one."""
    cfg = fh.synth.vabirax_config(40, 50, [fh.synth.vabirax_layer(2, 16, 8, 16, 24, 32, 30, 50), fh.synth.vabirax_layer(1, 16, 8, 16, 24, 32, None, None)],
                                  loop=(0, 1, 2))
    c = Case(fh, vo, tmp_path, cfg)
    ids = c.ids(4160, seed=51)
    want = c.oracle.forward(ids)[0]
    m = c.model(max_seq=4224)
    rows = np.r_[0, 2000, 4090:4160]
    check(m.prefill_logits(ids, rows), want[rows], "float32")
    check(m.forward(7), c.oracle.forward(np.r_[ids, 7])[0][-1], "float32")
    m.close()


# ---- one mechanism at a time ------------------------------------------------------------------------------------------------------

def silenced(tensors, fh, *names):
    """The post-norm of these sublayers without weight and bias: the sublayer adds nothing."""
    t = dict(tensors)
    for n in names:
        t[n], t[n + ".b"] = np.zeros_like(t[n]), np.zeros_like(t[n + ".b"])
    return t


def test_mechanisms_alone(fh, vo, torch_gpu, tmp_path):
    lay = fh.synth.vabirax_layer(3, 12, 6, 10, 14, 18, 25, 11)
    cfg = fh.synth.vabirax_config(50, 60, [lay], embedding_scale=2.5, eps=0.02)
    looped = fh.synth.vabirax_config(50, 60, [lay], loop=(0, 1, 1), embedding_scale=2.5, eps=0.02)
    base = fh.synth.folder_tensors(looped, 8)
    f = {k: fh.synth.from_bf16(v).astype(np.float64) for k, v in base.items()}
    norm = lambda x, n: vo.dyn_tanh(x, f[n + ".alpha"], f[n], f[n + ".b"])
    part = lambda prefix: {k[len(prefix):]: v for k, v in f.items() if k.startswith(prefix)}
    ids = np.random.default_rng(5).integers(0, 60, 90)
    x0 = f["embed"][ids] * 2.5
    plain = {k: v for k, v in base.items() if k != "loop.in"}

    def residual(name, config, tensors):
        c = Case(fh, vo, tmp_path / name, config, tensors)
        m = c.model()
        out = m.prefill_residuals(ids)[0]
        m.close()
        return out

    # the embedding and its scale
    check(residual("embedding", cfg, silenced(plain, fh, "l0.norm1b", "l0.norm2b")), x0, "float32")
    # the loop's input product
    got = residual("loop", looped, silenced(base, fh, "l0.norm1b", "l0.norm2b"))
    check(got, vo.loop_input(x0, x0, f["loop.in"]), "float32")
    # latent attention behind its norms
    a = norm(vo.latent_attention(norm(x0, "l0.norm1"), part("l0.mix."), lay["mixer"], 0.02), "l0.norm1b")
    check(residual("attention", cfg, silenced(plain, fh, "l0.norm2b")) - x0, a, "float32")
    # the feed-forward behind its norms
    b = norm(vo.gated_ff(norm(x0, "l0.norm2"), part("l0.mlp.")), "l0.norm2b")
    check(residual("ff", cfg, silenced(plain, fh, "l0.norm1b")) - x0, b, "float32")
    # the post-norm of a sublayer that computes nothing is its bias
    t = dict(plain)
    t["l0.mix.o"] = np.zeros_like(t["l0.mix.o"])
    check(residual("bias", cfg, silenced(t, fh, "l0.norm2b")) - x0, np.broadcast_to(f["l0.norm1b.b"], x0.shape), "float32")


@pytest.mark.parametrize("M,N,K", [(1, 1, 64), (1, 203, 448), (1, 4096, 2048), (1, 13001, 1088), (1, 96, 8192), (2, 5, 64), (33, 130, 192), (64, 64, 64), (65, 67, 1024),
                                   (200, 4100, 128), (1500, 2050, 320)])
def test_dense_products(fh, torch_gpu, M, N, K):
    torch = torch_gpu
    print("dense", M, N, K, flush=True)
    g = torch.Generator().manual_seed(M + N + K)
    a, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g)
    for name, code, limit in ((torch.float32, fh.F32, 2e-6), (torch.bfloat16, fh.BF16, 2e-6)):
        ad, wd = a.to(name).cuda(), w.to(name).cuda()
        y = torch.full((M, N), float("nan"), device="cuda")
        fh.check(fh.lib().forge_hip_dense_matmul(code, wd.data_ptr(), ad.data_ptr(), M, N, K, y.data_ptr(), None))
        torch.cuda.synchronize()
        want = ad.cpu().double() @ wd.cpu().double().T
        assert (y.cpu().double() - want).abs().max() <= limit * K ** 0.5 * 4
    for bad in ((0, 4, 64), (4, 4, 96), (4, 4, 0)):
        with pytest.raises(fh.ForgeHipError):
            fh.check(fh.lib().forge_hip_dense_matmul(fh.F32, wd.data_ptr(), ad.data_ptr(), *bad, y.data_ptr(), None))


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
    # temperature and the repeat penalty go through the shared sampler: a penalised greedy run differs, and is repeatable
    runs = []
    for _ in range(2):
        m.reset()
        runs.append(m.generate(prompt, max_tokens=24, repeat_penalty=1.3))
    ids, out = [int(t) for t in prompt], []
    logits = c.oracle.forward(ids)[0][-1]
    for _ in range(24):
        nxt = int(np.flatnonzero(logits == logits.max())[-1])
        out.append(nxt)
        ids.append(nxt)
        logits = c.oracle.forward(ids)[0][-1]
        for t in ids:
            logits[t] = logits[t] / 1.3 if logits[t] > 0 else logits[t] * 1.3
    assert runs[0] == runs[1] == out
    m.reset()
    m.set_repeat_penalty(1.0)
    sampled = m.generate(prompt, max_tokens=12, temperature=0.8, repeat_penalty=1.0, seed=77)
    m.reset()
    assert m.generate(prompt, max_tokens=12, temperature=0.8, repeat_penalty=1.0, seed=77) == sampled
    m.close()


def test_chat_server_serves_the_model(get, fh):
    c = get("no_window")

    class Ids:
        """A tokenizer of one token per character."""
        def encode(self, text, add_special_tokens):
            return [ord(ch) % 150 for ch in text]

        def decode(self, ids, skip_special_tokens):
            return "<%d>" % ids[0]

    m = c.model()
    body = json.dumps({"messages": [{"role": "user", "content": "hello"}], "max_tokens": 6}).encode()
    status, _, answer = fh.serve.ChatServer(m, Ids()).handle("POST", "/v1/chat/completions", body)
    assert status == 200
    prompt = Ids().encode(fh.serve.format_chat_messages([{"role": "user", "content": "hello"}]), True)
    want = c.oracle.greedy(prompt, 6)
    want = want[:want.index(2)] if 2 in want else want
    assert json.loads(answer)["choices"][0]["message"]["content"] == "".join("<%d>" % t for t in want)
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
    assert pre["gate_up_matmul"][1] == 4 and pre["attention"][1] == 6              # runs: 0 | 1 2 | 1 2 | 3, layer 1 without a feed-forward
    m.close()


def test_other_number_formats_and_refusals(get, fh, vo, tmp_path):
    c = get("part_rotation")
    # 32-bit tensors in the file: the float32 model takes them as they are
    rng = np.random.default_rng(4)
    t = {k: (fh.synth.from_bf16(v) * (1 + 1e-3 * rng.standard_normal(v.shape))).astype(np.float32) for k, v in c.tensors.items()}
    f = Case(fh, vo, tmp_path / "f32", c.cfg, t)
    ids = f.ids(40)
    m = f.model()
    check(m.prefill_logits(ids, np.arange(40)), f.oracle.forward(ids)[0], "float32")
    with pytest.raises(fh.ForgeHipError, match="K/V cache"):
        m._check(m._lib.forge_hip_model_read_kv(m._h, 0, 0, np.empty(16, np.uint16).ctypes.data))
    m.reset()
    with pytest.raises(fh.ForgeHipError, match="flat cache"):
        m.set_kv_pages(64, np.arange(4))
    with pytest.raises(fh.ForgeHipError):
        m.forward_prefill_batch([c.cfg["vocab"]])
    with pytest.raises(fh.ForgeHipError):
        m.prefill_logits(ids[:4], [4])
    m.close()
    m = fh.HipModel.from_path(f.path, 64, dtype="bfloat16")
    assert m.config["max_seq"] == 64 and m.config["wdtype"] == fh.BF16
    m.close()
    for name, change in (("missing", lambda t: t.pop("l0.mix.uv")), ("shape", lambda t: t.update({"l0.mix.o": t["l0.mix.o"][:, :-1]})),
                         ("alpha", lambda t: t.update({"final.norm.alpha": np.zeros(1, np.uint16)}))):
        bad = dict(c.tensors)
        change(bad)
        fh.synth.write_model_folder(str(tmp_path / name), c.cfg, bad)
        with pytest.raises(fh.ForgeHipError, match="tensor"):
            fh.HipModel.from_folder(str(tmp_path / name), 64)
    big = json.loads(json.dumps(c.cfg))
    big["layers"][0]["mixer"]["kv_rank"] = 1100
    fh.synth.write_model_folder(str(tmp_path / "big"), big, fh.synth.folder_tensors(big, 1))
    with pytest.raises(fh.ForgeHipError, match="kv_rank"):
        fh.HipModel.from_folder(str(tmp_path / "big"), 64)


def test_command_line(get):
    c = get("uneven")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompt = c.ids(12, seed=62)
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), c.path, "--ids", ",".join(map(str, prompt)), "--max-tokens", "9",
                        "--repeat-penalty", "1", "--dtype", "float32"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split()[-1].split(",")] == c.oracle.greedy(prompt, 9)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(get, tmp_path, dtype):
    """bin/trace_run on a small trace: two requests, one after the other, prompt portions and single tokens."""
    c = get("uneven")
    replay(c, {"a": c.ids(70, seed=71), "b": c.ids(33, seed=72)}, (40, 1, 2, 1, 1000), dtype, tmp_path)
