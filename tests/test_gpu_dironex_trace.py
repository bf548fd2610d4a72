"""bin/trace_run end to end on a Dironex directory of the test's own making: the command line picks the model class by config.json, replays steps (whole prompts,
prompt + decoded tokens, a batch of unequal requests decoded together, states given back and reused) and writes the logits asked for -- against the float64 oracle,
in both precisions."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import dironex_oracle as O

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def model(tmp_path):
    cfg = O.config(vocab=83, width=48, eps=3e-6, taps=4, streams=2, mult=0.45, embed_scale=0.8, loop=(1, 3, 2), layers=[
        O.attention_layer(6, 3, 8, 16, window=50, scale=0.3, mlp=O.moe(9, 2, 12, (3, 1), 1.4)),
        O.latent_layer(3, 16, 8, 16, 32, 20, O.rot(8, 3000.0, O.yarn(2.0, 64, 16.0, 1.0)), scale=0.2, mlp=O.dense(24)),
        O.attention_layer(2, 1, 24, 8, window=13, mlp=None),
        O.latent_layer(2, 8, 16, 8, 16, 24, O.rot(16), mlp=O.moe(6, 3, 16, (2, 2), 2.0)),
    ])
    W = O.weights(cfg, 17)
    path = str(tmp_path / "model")
    O.write_model_dir(path, cfg, W)
    return cfg, {k: v.astype(np.float64) for k, v in W.items()}, path


def replay(path, dtype, steps, out):
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", out, "--max-tokens", "700"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    done = [l for l in p.stdout.splitlines() if l.startswith("done ")]
    assert done == [f"done {s['step']}" for s in steps]
    return {s["step"]: np.fromfile(os.path.join(out, f"{s['step']}.f32"), dtype="<f4") for s in steps if any(e.get("want") for e in s["entries"])}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner_whole_decode_and_together(tmp_path, dtype):
    cfg, W, path = model(tmp_path)
    V = cfg["vocab"]
    rng = np.random.default_rng(4)
    reqs = {name: [int(t) for t in rng.integers(0, V, size=n)] for name, n in (("a", 150), ("b", 1), ("c", 67), ("d", 40))}
    want = {k: O.forward(cfg, W, t)[0] for k, t in reqs.items()}
    steps, expect = [], {}

    def step(entries, end=(), rows=None):
        steps.append({"step": len(steps), "entries": entries, "end": list(end)})
        if rows is not None:
            expect[len(steps) - 1] = np.asarray(rows)
    # a: whole, every tenth position asked for; its state goes back and is taken by the next request
    step([{"id": "a", "tokens": reqs["a"], "want": list(range(0, 150, 10))}], ["a"], want["a"][0:150:10])
    # c: most of the prompt, then token by token over the windows' edges
    step([{"id": "c", "tokens": reqs["c"][:39], "want": [38]}], (), want["c"][38:39])
    for i in range(39, 67):
        step([{"id": "c", "tokens": [reqs["c"][i]], "want": [0] if i % 2 else []}], ["c"] if i == 66 else [], want["c"][i:i + 1] if i % 2 else None)
    # b, d and a again (another name) together, unequal lengths; then decoded together, the short ones leaving first
    cut = {"b": 1, "d": 30, "e": 140}
    reqs["e"], want["e"] = reqs["a"], want["a"]
    step([{"id": k, "tokens": reqs[k][:cut[k]], "want": [cut[k] - 1]} for k in ("b", "d", "e")], ["b"], [want[k][cut[k] - 1] for k in ("b", "d", "e")])
    for i in range(10):
        live = [k for k in ("d", "e") if cut[k] + i < len(reqs[k])]
        step([{"id": k, "tokens": [reqs[k][cut[k] + i]], "want": [0]} for k in live], [k for k in live if cut[k] + i == len(reqs[k]) - 1], [want[k][cut[k] + i] for k in live])
    got = replay(path, dtype, steps, str(tmp_path / "out"))
    assert sorted(got) == sorted(expect)
    errs = np.concatenate([O.logit_error(got[n].reshape(-1, V), expect[n].reshape(-1, V)) for n in sorted(expect)])
    if dtype == "float32":
        assert errs.max() < 4e-5, errs.max()
    else:  # the rounding noise of bf16 products in a narrow stream: a row may stand out
        assert np.median(errs) < 3e-2 and np.mean(errs < 6e-2) >= 0.9, (np.median(errs), errs.max())
