"""The command line: one dispatcher, one function per command (reference lockstep:32-95).
The commands that need no GPU are run here as subprocesses; the others in test_cli_gpu.py."""

from __future__ import annotations

import json
import subprocess
import sys
from pathlib import Path

ROOT = Path(__file__).resolve().parent.parent
LOCKSTEP = [sys.executable, str(ROOT / "bin" / "lockstep")]


def run(*args, **kw):
    return subprocess.run([*LOCKSTEP, *args], capture_output=True, text=True, timeout=300, **kw)


def test_help_lists_every_command_and_says_what_is_not_built():
    done = run("--help")
    assert done.returncode == 0
    for name in ("run", "replay", "bench", "init", "verify", "certify"):
        assert name in done.stdout
    assert "not built" in done.stdout
    assert run().returncode == 0


def test_unknown_and_unbuilt_commands_exit_with_2():
    assert run("frobnicate").returncode == 2
    done = run("certify")
    assert done.returncode == 2 and "not built" in done.stdout


def test_init_writes_a_model_folder_from_a_preset_and_from_a_config(tmp_path):
    from lockstep_amd.config import config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "tiny-b", "--out", str(tmp_path / "b"), "--seed", "4", "--norm-std", "0.1")
    assert done.returncode == 0, done.stderr
    assert done.stdout.strip() == str(tmp_path / "b")
    config = config_from_dir(tmp_path / "b")
    assert config.hidden_size == 96 and not config.tie_word_embeddings
    names = SafetensorsFile(tmp_path / "b" / "model.safetensors").keys()
    assert "lm_head.weight" in names and "model.layers.2.self_attn.q_norm.weight" in names
    raw = json.loads((tmp_path / "b" / "config.json").read_text())
    raw["num_hidden_layers"] = 1
    (tmp_path / "one.json").write_text(json.dumps(raw))
    done = run("init", "--config", str(tmp_path / "one.json"), "--out", str(tmp_path / "c"))
    assert done.returncode == 0, done.stderr
    assert config_from_dir(tmp_path / "c").num_hidden_layers == 1
    assert run("init", "--preset", "no-such", "--out", str(tmp_path / "d")).returncode != 0


def test_run_needs_prompts_and_a_model():
    assert run("run", "--random", "tiny-a").returncode == 2          # no prompts
    assert run("run", "--prompt-ids", "1 2 3").returncode == 2       # neither --model nor --random


def test_init_writes_a_bikovik_folder_from_its_preset(tmp_path):
    from lockstep_amd.config import BikovikConfig, config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "bikovik-tiny", "--out", str(tmp_path / "k"), "--seed", "2")
    assert done.returncode == 0, done.stderr
    config = config_from_dir(tmp_path / "k")
    assert isinstance(config, BikovikConfig) and config.width == 128 and len(config.layers) == 4
    names = SafetensorsFile(tmp_path / "k" / "model.safetensors").keys()
    for name in ("embed", "head", "final.norm.alpha", "l0.mix.lower", "l1.mix.talk", "l3.mix.vmix", "l2.mix.g", "l2.mlp.down"):
        assert name in names, name


def test_init_writes_a_biberax_folder_from_its_preset(tmp_path):
    from lockstep_amd.config import BiberaxConfig, config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "biberax-tiny", "--out", str(tmp_path / "k"), "--seed", "2")
    assert done.returncode == 0, done.stderr
    config = config_from_dir(tmp_path / "k")
    assert isinstance(config, BiberaxConfig) and config.width == 128 and len(config.layers) == 4
    handle = SafetensorsFile(tmp_path / "k" / "model.safetensors")
    names = handle.keys()
    for name in ("embed", "head", "final.norm", "l0.mix.g", "l0.mlp.gate", "l1.mix.rel", "l1.mix.sink", "l1.mix.q.norm",
                 "l1.mlp.e7.down", "l1.mlp.router.b", "l2.mlp.shared.up", "l3.mix.o.b"):
        assert name in names, name
    assert "l1.mix.v" not in names and "l3.mlp.gate" not in names
    assert tuple(handle.shape("l1.mix.rel")) == (16, 4)


def test_init_writes_a_toripel_folder_from_its_preset(tmp_path):
    from lockstep_amd.config import ToripelConfig, config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "toripel-tiny", "--out", str(tmp_path / "k"), "--seed", "2")
    assert done.returncode == 0, done.stderr
    config = config_from_dir(tmp_path / "k")
    assert isinstance(config, ToripelConfig) and config.width == 128 and len(config.layers) == 4 and config.streams == 2
    handle = SafetensorsFile(tmp_path / "k" / "model.safetensors")
    names = handle.keys()
    for name in ("embed", "head", "final.norm", "l0.mix.q.conv", "l0.mix.A_log", "l0.hc1.mix", "l0.hc2.in", "l0.mlp.table",
                 "l0.mlp.e7.down", "l1.mix.k.b", "l2.mix.dkv", "l2.mix.dkv.norm", "l2.mix.sink", "l3.mix.uk", "l3.mix.dq.norm"):
        assert name in names, name
    assert "l3.mix.dkv" not in names and "l3.mlp.table" not in names and "l0.mlp.router" not in names
    assert tuple(handle.shape("l0.mlp.table")) == (640, 2) and tuple(handle.shape("l2.mix.dkv")) == (48, 128)


def test_init_writes_a_narurax_folder_from_its_preset(tmp_path):
    from lockstep_amd.config import NaruraxConfig, config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "narurax-tiny", "--out", str(tmp_path / "k"), "--seed", "2")
    assert done.returncode == 0, done.stderr
    config = config_from_dir(tmp_path / "k")
    assert isinstance(config, NaruraxConfig) and config.width == 128 and len(config.layers) == 4
    handle = SafetensorsFile(tmp_path / "k" / "model.safetensors")
    names = handle.keys()
    for name in ("embed", "bigram", "head", "final.norm", "l0.shift", "l3.shift", "l0.mix.q.conv", "l0.mix.A_log", "l0.mix.a1",
                 "l0.mix.g2", "l0.mlp.router", "l0.mlp.e7.down", "l1.mix.talk", "l1.mix.sink", "l1.mix.g", "l2.mix.q.norm",
                 "l2.mix.k.b", "l2.mix.o.b"):
        assert name in names, name
    assert "l1.mix.v" not in names and "l3.mlp.router" not in names and "l0.mlp.router.b" not in names and "l0.mix.a" not in names
    assert tuple(handle.shape("bigram")) == (510, 128) and tuple(handle.shape("l0.mix.dt_bias")) == (128,)


def test_init_writes_a_tukavik_folder_from_its_preset(tmp_path):
    from lockstep_amd.config import TukavikConfig, config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "tukavik-tiny", "--out", str(tmp_path / "k"), "--seed", "2")
    assert done.returncode == 0, done.stderr
    config = config_from_dir(tmp_path / "k")
    assert isinstance(config, TukavikConfig) and config.width == 128 and len(config.layers) == 4
    handle = SafetensorsFile(tmp_path / "k" / "model.safetensors")
    names = handle.keys()
    for name in ("embed", "final.norm", "l0.norm1", "l0.norm1b", "l0.norm2b", "l0.mix.z.b", "l0.mix.g", "l0.mlp.act", "l0.dwa",
                 "l1.mix.q", "l1.mix.dkv.norm", "l1.mix.uv", "l3.mix.dq.norm", "l3.mix.uq", "l3.dwa"):
        assert name in names, name
    assert "head" not in names and "l3.mix.dkv" not in names and "l2.mlp.up" not in names and "l1.mix.dq" not in names
    assert tuple(handle.shape("l3.dwa")) == (5,) and tuple(handle.shape("l1.mix.dkv")) == (40, 128)


def test_init_writes_a_pozozen_folder_from_its_preset(tmp_path):
    from lockstep_amd.config import PozozenConfig, config_from_dir
    from lockstep_amd.weights import SafetensorsFile

    done = run("init", "--preset", "pozozen-tiny", "--out", str(tmp_path / "k"), "--seed", "2")
    assert done.returncode == 0, done.stderr
    config = config_from_dir(tmp_path / "k")
    assert isinstance(config, PozozenConfig) and config.width == 128 and config.order() == [0, 1, 2, 1, 2, 3]
    handle = SafetensorsFile(tmp_path / "k" / "model.safetensors")
    names = handle.keys()
    for name in ("embed", "head", "final.norm", "final.norm.b", "l0.norm1.b", "l0.hc1.mix", "l0.mix.left.q.b", "l0.mix.right.in",
                 "l0.mix.right.conv.b", "l0.mix.right.A_log", "l0.mlp.correction", "l0.mlp.e7.up", "l0.mlp.shared.down", "l1.mix.i.b",
                 "l1.mix.norm", "l3.mix.g"):
        assert name in names, name
    assert "l0.mlp.e8.up" not in names and "l3.mlp.router" not in names and "l1.mix.left.q" not in names
    assert tuple(handle.shape("l0.mlp.router")) == (10, 128) and tuple(handle.shape("l0.mix.right.conv")) == (256, 4)
