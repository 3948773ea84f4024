"""Povazen's host side without a GPU: configuration and registry, the per-layer state's books, argument checks of the
entry points, the trace replay's handling of requests."""

import ctypes
import json
import os

import pytest
import torch

from _povazen import CONFIGS
from ohara_amd import _lib, build
from ohara_amd.checkpoint import ARCHITECTURES, _architecture, load_checkpoint
from ohara_amd.povazen import Povazen, PovazenConfig
from ohara_amd.state_cache import LayerState


def test_config_from_json_and_registry(tmp_path):
    from safetensors.torch import save_file

    save_file({"embed": torch.zeros(2, 2, dtype=torch.bfloat16)}, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    cfg, state = load_checkpoint(tmp_path, max_sequence_length=77)
    assert isinstance(cfg, PovazenConfig) and list(state) == ["embed"]
    assert (cfg.vocab_size, cfg.hidden_size, cfg.conv_taps, cfg.norm_groups, cfg.logit_softcap) == (97, 60, 4, 3, 12.0)
    assert cfg.max_sequence_length == 77 and cfg.num_hidden_layers == 4
    assert [(l.type, l.heads, l.kv_heads, l.dim, l.vdim, l.conv, l.ff) for l in cfg.layers[:2]] == [
        ("channel_delta", 4, 2, 24, 20, 2, 44), ("attention", 6, 2, 20, 12, 0, 0)]
    assert cfg.layers[1].scale == 0.3
    assert load_checkpoint(tmp_path)[0].max_sequence_length == PovazenConfig.max_sequence_length
    assert PovazenConfig.from_dict(CONFIGS["ones"]).logit_softcap == 0.0
    assert _architecture("Povazen") == (PovazenConfig, Povazen)


@pytest.mark.parametrize("change, message", [
    (dict(layers=[{"type": "window", "mixer": {"heads": 1, "kv_heads": 1, "dim": 8, "vdim": 8}, "mlp": None}]), "unknown mixer"),
    (dict(layers=[dict(CONFIGS["odd"]["layers"][0], mlp={"kind": "experts", "ff": 8})]), "unknown feed-forward"),
])
def test_config_rejects_what_it_does_not_know(change, message):
    with pytest.raises(ValueError, match=message):
        PovazenConfig.from_dict({**CONFIGS["odd"], **change})


def test_layer_state_books():
    st = LayerState(16, {"key": torch.zeros(3, 16, 2), "conv": torch.zeros(3, 4)}, idx=5)
    assert st.idx == 5 and st.capacity == 3 and st.key.shape == (3, 16, 2) and not st.int8
    with pytest.raises(AttributeError):
        st.value
    st._commit(3, st._reserve(3, 4, 0))
    with pytest.raises(ValueError, match="sequential"):
        st._reserve(3, 1, 5)
    with pytest.raises(ValueError, match="exceeds"):
        st._reserve(3, 13, 4)
    assert st._reserve_ragged(3, [1, 2, 3], [4, 4, 4]) == [5, 6, 7]
    st._commit_ragged(3, [5, 6, 7])
    assert st._reserve_rows([2, 0], [1, 1], [7, 5]) == [8, 6]
    st._commit_rows([2, 0], [8, 6])
    assert st.lengths == [6, 6, 8] and st.length == 8
    for slots in ([0, 0], [3, 1], [-1, 0]):
        with pytest.raises(ValueError, match="slots"):
            st._reserve_rows(slots, [1, 1], [6, 6])
    with pytest.raises(ValueError, match="sequential"):
        st._reserve_rows([1], [1], [5])
    view = st._row_view(2)
    assert view.length == 8 and view.capacity == 1 and view.key.data_ptr() == st.key[2:].data_ptr()


def test_entry_points_check_their_arguments():
    L = _lib.lib()
    assert ctypes.sizeof(_lib.OharaSeq) == 4 * 4 + 3 * 8
    assert ctypes.sizeof(_lib.OharaDelta) == 12 * 4 + 6 * 8 and _lib.OharaDelta.conv_w.offset == 48
    seq = _lib.OharaSeq(1, 1, 0, 0, None, None, None)
    two = _lib.OharaSeq(1, 2, 0, 0, None, None, None)
    r = ctypes.byref
    buf = ctypes.create_string_buffer(4096)
    p = ctypes.addressof(buf)
    assert L.ohara_residual_norm_bf16(0, 8, 0, 0, 0, 1.0, 0, 0, 0, 1, 1e-5, 0, 0, 0, 0, 0, 0, 0, None, r(seq), 0) == _lib.EINVAL
    # groups do not divide the width; the fused convolution takes one token per sequence
    assert L.ohara_residual_norm_bf16(p, 8, 0, 0, 0, 1.0, p, 8, p, 3, 1e-5, 0, 0, 0, 0, 0, 0, 0, None, r(seq), 0) == _lib.EINVAL
    assert L.ohara_residual_norm_f32(p, 8, 0, 0, 0, 1.0, p, 8, p, 1, 1e-5, 2, p, 8, 0, p, 2, p, None, r(two), 0) == _lib.EINVAL
    assert L.ohara_attn_bias_bf16(p, p, p, 2, 1, 300, 8, 16, 1.0, p, 0, 0, 1, 0, p, 16, r(seq), 0) == _lib.ESIZE
    assert L.ohara_attn_bias_bf16(p, p, p, 3, 2, 8, 8, 16, 1.0, p, 0, 0, 1, 0, p, 24, r(seq), 0) == _lib.EINVAL
    assert L.ohara_attn_bias_bf16(p, p, p, 2, 1, 8, 8, 16, 1.0, p, 0, 0, 2, 0, p, 16, r(seq), 0) == _lib.EINVAL  # no workspace
    late = _lib.OharaSeq(1, 1, 16, 0, None, None, None)
    assert L.ohara_attn_bias_f32(p, p, p, 2, 1, 8, 8, 16, 1.0, p, 0, 0, 1, 0, p, 16, r(late), 0) == _lib.EINVAL  # past the cache
    assert L.ohara_gemm_f32(p, 6, p, 0, 0, 0.0, 4, 6, 1, p, 4, 0) == _lib.EINVAL  # k % 4
    assert L.ohara_gemm_softcap_bf16(p, 8, p, 8, 8, 0.0, 1, p, 8, 0) == _lib.EINVAL
    d = _lib.OharaDelta()
    assert L.ohara_delta_step_f32(r(d), p, 8, p, p, p, 8, r(seq), 0) == _lib.EINVAL
    assert L.ohara_delta_workspace_bytes(1, 300, 8, 1, 1) == _lib.EINVAL
    assert L.ohara_delta_workspace_bytes(2, 40, 24, 3, 33) == 4 * 2 * 3 * 2 * (3 * 32 * 64 + 32 * 32 + 32 * 32 + 64)


def test_partial_library_sources_exist():
    names = {os.path.basename(s)[:-4] for s in build.sources()}
    assert set().union(*build.SERVING.values()) <= names and set(build.SERVING) == set(ARCHITECTURES)


class _Model:
    """A model that answers with the ids it was fed and the positions they sat at."""

    supports_seq_lens = True
    device = torch.device("cpu")

    class config:
        max_sequence_length, vocab_size = 32, 4

    def __init__(self):
        self.calls = []

    def build_kv_cache(self, batch_size=1, int8=False):
        return [LayerState(32, {"s": torch.zeros(batch_size, 1)})]

    def forward(self, x, cache, positions, *, last_only=False, seq_pos=None, seq_lens=None, slots=None):
        B, S = x.shape
        self.calls.append((x.tolist(), list(positions), seq_lens, slots))
        out = torch.zeros(B, S, 4)
        out[..., 0] = x
        out[..., 1] = torch.tensor(positions).view(B, 1) + torch.arange(S)
        return out[:, -1:] if last_only else out


def test_replay_runs_the_batcher_and_gives_slots_back():
    from ohara_amd.trace import Replay

    m = _Model()
    r = Replay(m)
    a, b = r.step([("a", [5, 6, 7]), ("b", [8])])
    assert a[:, 0].tolist() == [5, 6, 7] and a[:, 1].tolist() == [0, 1, 2] and b.shape == (1, 4)
    assert m.calls[-1][0] == [[5, 6, 7], [8, 0, 0]] and m.calls[-1][2:] == ([3, 1], [0, 1])
    b, a = r.step([("b", [9]), ("a", [4])])
    assert m.calls[-1] == ([[4], [9]], [3, 1], None, None)  # the decode step of every slot
    assert a[0, :2].tolist() == [4, 3] and b[0, :2].tolist() == [9, 1]
    r.end("a")
    (b,) = r.step([("b", [3])])
    assert m.calls[-1] == ([[0], [3]], [0, 2], None, None) and b[0, :2].tolist() == [3, 2]
    assert r.batcher.lengths == [0, 3]
    (b,) = r.step([("b", [1, 2])])  # a portion of a continued request
    assert m.calls[-1] == ([[1, 2]], [3], [2], [1]) and b[:, 1].tolist() == [3, 4]
    r.end("b")
    assert r.batcher.free_slots() == [0, 1]
    r.step([("c", [1])])
    assert r.batcher.slots == 1 and r.batcher.lengths == [1]
    with pytest.raises(RuntimeError, match="no free slot"):
        r.step([("c", [1]), ("d", [1])])
