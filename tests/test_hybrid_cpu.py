"""Host side of the decoders chosen by configuration: the registry, what it refuses, the C ABI's checks, the plain statement's
own consistency.  Nothing here touches a GPU."""
import ctypes as C
import json
import os
import re
import subprocess
import sys

import numpy as np
import pytest

import hybrid_models as hm
import plain_hybrid as ph
import ug_amd

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_layer_entry_points_are_exported_and_refuse_a_null_device():
    text = open(os.path.join(ROOT, "include", "ughip_layers.h")).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    names = sorted(set(re.findall(r"\bint (ughip_[a-z0-9_]+)\s*\(", text)))
    assert len(names) >= 14
    lib = ug_amd.ughip_lib()
    for n in names:
        fn = getattr(lib, n)
        fn.restype = C.c_int
    for n in ("ughip_product_rows", "ughip_product_row"):
        assert getattr(lib, n)(None, None) != 0 and "null" in lib.ughip_last_error().decode()
    assert lib.ughip_group_rows(None, None, C.c_size_t(1), C.c_size_t(1), C.c_size_t(1), None, None, None) != 0


def test_models_are_chosen_by_their_configuration(cpu, tmp_path):
    with pytest.raises(ug_amd.UgError, match="no model named 'Nothing'.*Tanolorn"):
        ug_amd.Decoder.random(cpu, {"architecture": "Nothing"})
    with pytest.raises(ug_amd.UgError, match="config.json"):
        ug_amd.Decoder.load(cpu, str(tmp_path / "absent"))
    llama = {"model_type": "llama", "hidden_size": 64, "intermediate_size": 96, "max_position_embeddings": 32, "num_attention_heads": 2, "num_hidden_layers": 1,
             "rms_norm_eps": 1e-5, "vocab_size": 50}
    assert ug_amd.Decoder.random(cpu, llama, bf16=False).vocab == 50
    assert ug_amd.Decoder.random(cpu, hm.ODD, bf16=False).vocab == hm.ODD["vocab"]


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="other"), "unknown mixer 'other'"),
    (lambda c: c["layers"][3]["mlp"].update(kind="other"), "unknown feed-forward 'other'"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "a router of 5 of 6"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "a router of"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "reads the latents of layer 0"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=4), "reads the latents of layer 4"),
    (lambda c: c["layers"][3]["mixer"].update(kv_rank=40), "none that fit"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=12), "rotates 12"),
    (lambda c: c.pop("width"), "'width' is missing"),
    (lambda c: c["layers"][0]["mixer"].update(heads="six"), "'heads' is not"),
])
def test_configurations_that_make_no_model_are_refused(cpu, change, message):
    cfg = json.loads(json.dumps(hm.ODD))
    change(cfg)
    with pytest.raises(ug_amd.UgError, match=message):
        ug_amd.Decoder.random(cpu, cfg, bf16=False)


def test_a_tensor_of_another_shape_is_refused(cpu, tmp_path):
    w = hm.weights(hm.ONES, 3)
    w["l1.mix.uq"] = np.zeros((4, 1))
    with pytest.raises(ug_amd.UgError, match="l1.mix.uq"):
        ug_amd.Decoder.load(cpu, hm.write(tmp_path / "m", hm.ONES, w), bf16=False)


@pytest.mark.parametrize("cfg", [hm.ODD, hm.ONES])
def test_the_plain_statement_is_causal(cfg):
    """Logits of a prefix do not change with what follows (windows of nothing, states, caches: all causal)."""
    w = hm.weights(cfg, 5)
    tokens = np.arange(23) * 7 % cfg["vocab"]
    full, part = ph.forward(cfg, w, tokens), ph.forward(cfg, w, tokens[:9])
    np.testing.assert_allclose(full[:9], part, rtol=1e-10, atol=1e-12)


def test_plain_rotation_and_convolution_by_hand():
    x = np.array([[[1.0, 2.0, 3.0, 4.0, 9.0]]])
    out = ph.rotate_half(x, [2], 100.0, 4)       # pairs (0, 2) and (1, 3), angles 2 and 2 / 10
    np.testing.assert_allclose(out[0, 0], [np.cos(2) - 3 * np.sin(2), 2 * np.cos(.2) - 4 * np.sin(.2), 3 * np.cos(2) + np.sin(2), 4 * np.cos(.2) + 2 * np.sin(.2), 9.0])
    y = ph.causal_conv(np.array([[1.0], [10.0], [100.0]]), np.array([[2.0, 3.0]]), np.array([0.5]))
    np.testing.assert_allclose(y[:, 0], [3.5, 32.5, 320.5])
    chosen, wts = ph.route(np.array([1.0]), {"router": np.array([[0.0], [0.0], [0.0], [0.0]]), "correction": np.array([-3.0, -1.0, -2.0, -1.5])},
                           {"experts": 4, "top": 2, "groups": {"count": 2, "keep": 1}})
    assert chosen.tolist() == [3, 2] and wts.tolist() == [0.5, 0.5]     # the second pair is better in sum (-2.5 against -3)


def test_the_command_line_programs_explain_themselves():
    for name in ("trace_run", "generate"):
        p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", name), "--help"], capture_output=True, text=True)
        assert p.returncode == 0 and "--model" in p.stdout
