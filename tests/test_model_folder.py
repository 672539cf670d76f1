"""The model-folder reader: round trips, and every malformed file is an error (no GPU)."""
import json
import os

import numpy as np
import pytest

import lokinex_synth as S
from wick_amd import checkpoint as K
from wick_amd import model as M


def raw_folder(path, header, data=b"", config='{"architecture": "Lokinex"}'):
    os.makedirs(path, exist_ok=True)
    (path / "config.json").write_text(config)
    text = header if isinstance(header, bytes) else json.dumps(header).encode()
    (path / "model.safetensors").write_bytes(len(text).to_bytes(8, "little") + text + data)
    return str(path)


def test_round_trip(tmp_path):
    cfg = S.mixed()
    t = S.tensors(cfg)
    with K.ModelFolder(S.write(tmp_path / "m", cfg, t)) as f:
        assert f.architecture == "Lokinex" and f.config == cfg
        assert sorted(f.names()) == sorted(t)
        for name, want in t.items():
            dtype, got = f.tensor(name)
            assert got.shape == want.shape
            if dtype == K.I32:
                assert np.array_equal(got, want)
            else:
                assert dtype == K.BF16 and np.array_equal(K.from_bf16(got).reshape(want.shape), want.astype(np.float32))
        with pytest.raises(K.CheckpointError):
            f.tensor("no.such")


def test_registry_names_the_architecture():
    assert {"Lokinex", "Zirurax"} <= set(M.folder_architectures())


def test_escapes_and_metadata(tmp_path):
    head = b'{"__metadata__": {"a": "b"}, "caf\\u00e9\\n": {"dtype": "I32", "shape": [], "data_offsets": [0, 4]}}'
    with K.ModelFolder(raw_folder(tmp_path / "m", head, b"\x05\0\0\0")) as f:
        assert f.names() == ["café\n"] and int(f.tensor("café\n")[1]) == 5


ok = {"dtype": "BF16", "shape": [2, 3], "data_offsets": [0, 12]}


@pytest.mark.parametrize("header, data", [
    ({"a": {**ok, "data_offsets": [0, 14]}}, b"\0" * 12),          # past the file
    ({"a": {**ok, "data_offsets": [4, 0]}}, b"\0" * 12),           # backwards
    ({"a": {**ok, "shape": [2, 4]}}, b"\0" * 12),                  # range does not fit the shape
    ({"a": {**ok, "shape": [2, 1e300]}}, b"\0" * 12),              # overflowing shape
    ({"a": {**ok, "shape": [-2, -3]}}, b"\0" * 12),
    ({"a": {**ok, "dtype": "F64"}}, b"\0" * 48),                   # a type that is not read
    ({"a": {"dtype": "BF16", "shape": [2, 3]}}, b"\0" * 12),       # incomplete
    (b'{"a": {"dtype": "I32", "shape": [], "data_offsets": [0, 4]}, "a": {"dtype": "I32", "shape": [], "data_offsets": [0, 4]}}', b"\0" * 4),
    (b"[1, 2", b""), (b'{"a": tru}', b""), (b'{"a" 1}', b""), (b"{} x", b""), (b"[" * 100 + b"]" * 100, b""), (b"[]", b""),
])
def test_malformed_tensors_are_errors(tmp_path, header, data):
    with pytest.raises(K.CheckpointError):
        K.ModelFolder(raw_folder(tmp_path / "m", header, data))


def test_malformed_files_are_errors(tmp_path):
    with pytest.raises(K.CheckpointError):
        K.ModelFolder(str(tmp_path / "missing"))
    for config in ("", "{", '{"architecture": 3}', "{}", "nul"):
        with pytest.raises(K.CheckpointError):
            K.ModelFolder(raw_folder(tmp_path / "c", {}, b"", config))
    p = tmp_path / "short"
    p.mkdir()
    (p / "config.json").write_text('{"architecture": "Lokinex"}')
    for data in (b"", b"\x01\0\0", (1 << 40).to_bytes(8, "little") + b"{}"):
        (p / "model.safetensors").write_bytes(data)
        with pytest.raises(K.CheckpointError):
            K.ModelFolder(str(p))
