"""CPU: bin/trace_run's options, and that it fails loudly where there is no GPU."""
import os
import subprocess
import sys

import net_models as nm

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EXE = os.path.join(ROOT, "bin", "trace_run")


def test_help_and_missing_options():
    assert os.access(EXE, os.X_OK)
    r = subprocess.run([sys.executable, EXE, "--help"], capture_output=True, text=True, timeout=120)
    assert r.returncode == 0 and "--max-tokens" in r.stdout
    r = subprocess.run([sys.executable, EXE, "--out", "x"], capture_output=True, text=True, timeout=120)
    assert r.returncode == 2 and "--model" in r.stderr
    r = subprocess.run([sys.executable, EXE, "--model", "m", "--out", "x", "--dtype", "int8"], capture_output=True, text=True, timeout=120)
    assert r.returncode == 2


def test_no_gpu_is_an_error(tmp_path):
    cfg = nm.MODELS["tiny"]
    path = nm.write(tmp_path / "m", cfg, nm.weights(cfg, 1))
    env = dict(os.environ, HIP_VISIBLE_DEVICES="-1", ROCR_VISIBLE_DEVICES="-1")
    r = subprocess.run([sys.executable, EXE, "--model", path, "--out", str(tmp_path)], input='{"step": 0, "entries": [], "end": []}\n', text=True,
                       capture_output=True, env=env, timeout=120)
    assert r.returncode not in (0, 3) and "done" not in r.stdout and "TgError" in r.stderr
