"""What the GPU tests of model folders share: a configuration with random weights on disk beside its plain restatement, and the
limits that its logits are held to.

float32: every operation is single precision, so logits agree to a few 1e-6 of their size: a wrong key, norm or rotation has
nowhere to hide.  bfloat16: the serving precision, held to the size of its rounding."""
import json
import os
import subprocess
import sys

import numpy as np

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LIMIT = {"float32": 3e-5, "bfloat16": 0.04}      # root mean square of a row's difference over that of all logits
DTYPES = list(LIMIT)


class Case:
    """A configuration with random weights on disk, its oracle, and handles to it."""

    def __init__(self, fh, plain, path, cfg, tensors=None, seed=5):
        self.fh, self.cfg, self.path = fh, cfg, str(path)
        self.tensors = tensors if tensors is not None else fh.synth.folder_tensors(cfg, seed)
        fh.synth.write_model_folder(self.path, cfg, self.tensors)
        self.oracle = plain.Oracle(cfg, {k: fh.synth.from_bf16(v) if v.dtype == np.uint16 else v for k, v in self.tensors.items()})

    def model(self, max_seq=256, dtype="float32"):
        return self.fh.HipModel.from_folder(self.path, max_seq, dtype)

    def ids(self, n, seed=9):
        return np.random.default_rng(seed).integers(0, self.cfg["vocab"], n)


def row_errors(got, want, scale=None):
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(want)
    assert np.all(np.isfinite(got))
    return np.sqrt(((got - want) ** 2).mean(axis=1)) / (scale or np.sqrt((want ** 2).mean()))


def check(got, want, dtype, scale=None):
    err = row_errors(got, want, scale)
    assert err.max() <= LIMIT[dtype], "row %d: %.3e" % (err.argmax(), err.max())


def decode_all(model, ids):
    return np.stack([model.forward(int(t)) for t in ids])


def replay(case, requests, portions, dtype, out):
    """bin/trace_run over the requests, each cut in `portions` (the last one: what is left); every answer against the oracle."""
    steps, expect = [], {}
    for name, ids in requests.items():
        want, at = case.oracle.forward(ids)[0], 0
        for n in portions:
            n = min(n, ids.size - at)
            if n <= 0:
                break
            rows = [] if n == 2 else sorted({0, n // 2, n - 1})[::-1]
            expect[len(steps)] = want[[at + r for r in rows]]
            steps.append({"step": len(steps), "entries": [{"id": name, "tokens": ids[at:at + n].tolist(), "want": rows}],
                          "end": [name] if at + n == ids.size else []})
            at += n
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", case.path, "--dtype", dtype, "--out", str(out), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [line for line in r.stdout.splitlines() if line.startswith("done")] == ["done %d" % i for i in range(len(steps))]
    scale = np.sqrt((case.oracle.forward(next(iter(requests.values())))[0] ** 2).mean())
    for i, want in expect.items():
        path = out / ("%d.f32" % i)
        assert path.exists() == (want.size > 0)
        if want.size:
            check(np.fromfile(path, "<f4").reshape(want.shape), want, dtype, scale)
