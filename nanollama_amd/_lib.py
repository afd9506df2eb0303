"""ctypes binding of the HIP libraries: libnanollama_hip.so (include/nanollama_hip.h, the quantised Llama family) and
libnanollama_stack.so (include/nanollama_stack.h, models described layer by layer).  Both export the same entry points on
handles of their own; a model class holds the library of its family and only that one is built and loaded.

The product path has no CPU fallback: if the HIP library is missing or no GPU is
visible, loading / creating a model raises.
"""
from __future__ import annotations

import ctypes as C
import os
import subprocess
import sys

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.environ.get("NL_LIB_PATH") or os.path.join(_HERE, "libnanollama_hip.so")  # NL_LIB_PATH: A/B builds (tools/)
STACK_LIB_PATH = os.environ.get("NL_STACK_LIB_PATH") or os.path.join(_HERE, "libnanollama_stack.so")
NL_NUM_KINDS = 11
NL_COMM_ID_BYTES = 128
NL_P2P_HANDLE_BYTES = 64
NL_FLAG_NO_GRAPH = 1
NL_FLAG_LOCAL_GROUP = 2
NL_FLAG_GROUP_FUSED = 4

STATUS = {0: "NL_OK", -1: "NL_ERR_INVALID", -2: "NL_ERR_UNSUPPORTED", -3: "NL_ERR_HIP", -4: "NL_ERR_STATE",
          -5: "NL_ERR_MISSING", -6: "NL_ERR_COMM"}


class NlConfig(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("n_layers", "dim", "n_heads", "n_kv_heads", "head_dim", "interm", "vocab",
                                         "seq_len")] + \
               [("rms_eps", C.c_float), ("rope_theta", C.c_float)] + \
               [(n, C.c_int32) for n in ("qk_norm", "rope_conjugate", "max_streams", "device", "tp_rank", "tp_size",
                                         "flags")]


class NlSampleParams(C.Structure):
    """nl_sample_params: the knobs of Engine.Generate's sampling branch (go/main.go:29-34, :135-140)."""
    _fields_ = [("temperature", C.c_float), ("top_p", C.c_float), ("top_k", C.c_int32), ("rep_penalty", C.c_float),
                ("rep_window", C.c_int32)]


class NlAttnDesc(C.Structure):
    """nl_attn_desc: the softmax-attention branch of a layer (heads == 0: none)."""
    _fields_ = [(n, C.c_int32) for n in ("heads", "kv_heads", "dim", "vdim", "window", "qk_norm", "distance_bias", "gate")] + \
               [("scale", C.c_float), ("mix_scale", C.c_float)]


class NlLinattnDesc(C.Structure):
    """nl_linattn_desc: the gated-linear-attention branch of a layer (heads == 0: none)."""
    _fields_ = [(n, C.c_int32) for n in ("heads", "dim", "vdim", "rank")] + [("tau", C.c_float), ("mix_scale", C.c_float)]


class NlLatentDesc(C.Structure):
    """nl_latent_desc: latent attention (heads == 0: none)."""
    _fields_ = [(n, C.c_int32) for n in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "kv_from", "rot_dims", "rot_adjacent", "sink", "gate")] + \
               [("scale", C.c_float)] + [(n, C.c_double) for n in ("rope_base", "yarn_factor", "yarn_original", "yarn_fast", "yarn_slow")]


class NlLayerDesc(C.Structure):
    _fields_ = [("attn", NlAttnDesc), ("lin", NlLinattnDesc), ("latent", NlLatentDesc)] + [(n, C.c_int32) for n in ("ff", "ff_act", "ff_bias")]


class NlStackConfig(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("vocab", "dim", "n_layers", "loop_start", "loop_stop", "loop_times", "seq_len", "max_streams",
                                         "max_step_tokens", "device", "dtype", "flags", "plain_norm", "post_norm", "untied")] + \
               [("eps", C.c_float), ("embed_scale", C.c_float)]


class NlError(RuntimeError):
    def __init__(self, code: int, msg: str):
        super().__init__(f"{STATUS.get(code, code)}: {msg}")
        self.code = code


_STACK_ONLY = ("nl_latent.h", "nl_linattn.h", "nl_mfma.h", "nl_winattn.h")
_STACK_HEADERS = ("nl_kernels.h", "nl_latent.h", "nl_linattn.h", "nl_mfma.h", "nl_sample.h", "nl_winattn.h")


def source_files(family: str = "hip"):
    """A library's sources in the order csrc/Makefile hashes them."""
    root, src_dir = os.path.dirname(_HERE), os.path.join(_HERE, "csrc")
    inc = lambda *names: [os.path.join(root, "include", n) for n in names]
    if family == "stack":
        return [os.path.join(src_dir, f) for f in ("nl_stack.hip",) + _STACK_HEADERS] + inc("nanollama_hip.h", "nanollama_stack.h")
    hdrs = sorted(f for f in os.listdir(src_dir) if f.endswith(".h") and f not in _STACK_ONLY)
    return [os.path.join(src_dir, f) for f in ["nl_engine.hip"] + hdrs] + inc("nanollama_hip.h")


def source_sha(files=None) -> str:
    import hashlib
    h = hashlib.sha256()
    for f in files or source_files():
        with open(f, "rb") as fh:
            h.update(fh.read())
    return h.hexdigest()[:16]


def build_info() -> dict:
    """What the loaded binary says it was built from, next to the sources present now."""
    L = lib()
    L.nl_build_info.restype = C.c_char_p
    info = dict(kv.split("=", 1) for kv in L.nl_build_info().decode().split())
    tree = source_sha()
    return {"lib_src_sha16": info.get("src"), "lib_git_head_at_build": info.get("git"), "tree_src_sha16": tree,
            "lib_matches_tree": info.get("src") == tree}


def build(force: bool = False, family: str = "hip") -> str:
    """Compile a family's HIP library for gfx950 in-tree (hipcc cross-compiles without a GPU).  Rebuilds when the binary is
    missing, older than a source, or carries another source hash than the tree (mtimes do not survive every copy)."""
    src_dir = os.path.join(_HERE, "csrc")
    path = LIB_PATH if family == "hip" else STACK_LIB_PATH
    files = source_files(family)
    stale = not os.path.exists(path) or any(os.path.getmtime(s) > os.path.getmtime(path) for s in files + [os.path.join(src_dir, "Makefile")])
    if not stale and not force:
        with open(path, "rb") as fh:       # read the embedded string without loading the library
            stale = f"src={source_sha(files)} git=".encode() not in fh.read()
    if force or stale:
        target = "../libnanollama_hip.so" if family == "hip" else "../libnanollama_stack.so"
        subprocess.check_call(["make", "-C", src_dir, "-B", target], stdout=sys.stderr)
    return path


_lib = None

EXPORTS = ["nl_build_info", "nl_set_gamma", "nl_abi_version", "nl_device_count", "nl_create", "nl_upload_tensor", "nl_finalize", "nl_destroy",
           "nl_last_error", "nl_reset", "nl_forward", "nl_forward_argmax", "nl_decode_greedy", "nl_prefill", "nl_forward_batch", "nl_get_config",
           "nl_synchronize", "nl_timer_start", "nl_timer_stop", "nl_kernel_kind_name", "nl_profile_forward",
           "nl_memory_usage", "nl_debug_read", "nl_op_matmul", "nl_op_matmul_batch", "nl_op_rmsnorm", "nl_comm_get_unique_id",
           "nl_comm_init", "nl_group_forward", "nl_debug_stamps", "nl_sample_decode", "nl_op_sample", "nl_p2p_export",
           "nl_p2p_import", "nl_p2p_info", "nl_p2p_loopback", "nl_op_exp", "nl_plan_info", "nl_persist_info", "nl_create_group", "nl_host_logits",
           "nl_op_gran16_soak"]


# what both families export (include/nanollama_stack.h lists it)
STACK_EXPORTS = ["nl_build_info", "nl_abi_version", "nl_device_count", "nl_create_stack", "nl_upload_tensor", "nl_finalize", "nl_destroy",
                 "nl_last_error", "nl_reset", "nl_forward", "nl_forward_argmax", "nl_decode_greedy", "nl_prefill", "nl_forward_batch",
                 "nl_get_config", "nl_synchronize", "nl_timer_start", "nl_timer_stop", "nl_memory_usage", "nl_debug_read",
                 "nl_sample_decode", "nl_host_logits", "nl_step", "nl_trace_layers"]

_vp, _i32, _fp, _ip = C.c_void_p, C.c_int, C.POINTER(C.c_float), C.POINTER(C.c_int)


def _bind_common(L):
    L.nl_abi_version.restype = _i32
    L.nl_device_count.restype = _i32
    L.nl_build_info.restype = C.c_char_p
    L.nl_upload_tensor.argtypes = [_vp, C.c_char_p, C.c_uint32, _vp, C.c_uint64, C.c_uint64, C.c_uint64]
    L.nl_finalize.argtypes = [_vp]
    L.nl_destroy.argtypes = [_vp]
    L.nl_last_error.restype = C.c_char_p
    L.nl_last_error.argtypes = [_vp]
    L.nl_reset.argtypes = [_vp, _i32]
    L.nl_forward.argtypes = [_vp, _i32, _i32, _i32, _fp]
    L.nl_forward_argmax.argtypes = [_vp, _i32, _i32, _i32, _ip]
    L.nl_decode_greedy.argtypes = [_vp, _i32, _i32, _i32, _i32, _ip, _ip]
    L.nl_prefill.argtypes = [_vp, _i32, _ip, _i32, _i32, _fp]
    L.nl_forward_batch.argtypes = [_vp, _ip, _ip, _ip, _i32, _fp, _ip]
    L.nl_get_config.argtypes = [_vp, C.POINTER(NlConfig)]
    L.nl_synchronize.argtypes = [_vp]
    L.nl_timer_start.argtypes = [_vp]
    L.nl_timer_stop.argtypes = [_vp, _fp]
    L.nl_memory_usage.argtypes = [_vp] + [C.POINTER(C.c_uint64)] * 3
    L.nl_debug_read.restype = C.c_int64
    L.nl_debug_read.argtypes = [_vp, C.c_char_p, _i32, _fp, C.c_int64]
    L.nl_host_logits.argtypes = [_vp]
    L.nl_host_logits.restype = _fp
    L.nl_sample_decode.argtypes = [_vp, _i32, _i32, _i32, C.POINTER(NlSampleParams), _fp, _ip, _ip, _ip, _ip]


def _open(path):
    if not os.path.exists(path):
        raise ImportError(f"{path} is missing: run `python -c 'import __graft_entry__ as g; g.build()'` "
                          "(the engine has no CPU fallback)")
    L = C.CDLL(path)
    _bind_common(L)
    return L


def lib():
    global _lib
    if _lib is not None:
        return _lib
    L = _open(LIB_PATH)
    vp, i32, fp, ip = _vp, _i32, _fp, _ip
    L.nl_create.argtypes = [C.POINTER(NlConfig), C.POINTER(vp)]
    L.nl_set_gamma.argtypes = [vp, C.POINTER(C.c_int32), i32, vp, i32]
    L.nl_kernel_kind_name.restype = C.c_char_p
    L.nl_kernel_kind_name.argtypes = [i32]
    L.nl_profile_forward.argtypes = [vp, i32, i32, i32, i32, fp, ip]
    L.nl_op_matmul.argtypes = [i32, C.c_uint32, vp, C.c_uint64, fp, fp, i32, i32]
    L.nl_op_matmul_batch.argtypes = [i32, C.c_uint32, vp, C.c_uint64, fp, fp, i32, i32, i32]
    L.nl_op_rmsnorm.argtypes = [i32, fp, fp, C.c_float, fp, i32]
    L.nl_comm_get_unique_id.argtypes = [vp]
    L.nl_comm_init.argtypes = [vp, vp]
    L.nl_p2p_export.argtypes = [vp, vp]
    L.nl_p2p_import.argtypes = [vp, vp]
    L.nl_p2p_info.argtypes = [vp, ip, ip]
    L.nl_p2p_loopback.argtypes = [vp]
    L.nl_plan_info.argtypes = [vp, ip, ip, ip, ip]
    L.nl_create_group.argtypes = [C.POINTER(NlConfig), ip, i32, C.POINTER(vp)]
    L.nl_persist_info.argtypes = [vp, ip, ip, C.POINTER(C.c_longlong), C.POINTER(C.c_longlong)]
    L.nl_op_exp.argtypes = [C.c_int, C.POINTER(C.c_float), C.POINTER(C.c_float), C.c_int]
    L.nl_op_gran16_soak.argtypes = [C.c_int, C.c_int, C.c_uint, C.POINTER(C.c_ulonglong), C.POINTER(C.c_ulonglong)]
    L.nl_group_forward.argtypes = [C.POINTER(vp), i32, i32, i32, i32, fp]
    L.nl_op_sample.argtypes = [i32, fp, i32, C.POINTER(NlSampleParams), C.c_float, ip, ip, ip]
    _lib = L
    return L


_stack = None


def stack_lib():
    """libnanollama_stack.so: the models described layer by layer."""
    global _stack
    if _stack is None:
        L = _open(STACK_LIB_PATH)
        L.nl_create_stack.argtypes = [C.POINTER(NlStackConfig), C.POINTER(NlLayerDesc), C.POINTER(_vp)]
        L.nl_step.argtypes = [_vp, _i32, _ip, _ip, _ip, _ip, _i32, _ip, _fp, _ip]
        L.nl_trace_layers.argtypes = [_vp, _i32]
        _stack = L
    return _stack


def check(handle, rc: int, L=None):
    if rc != 0:
        msg = (L or lib()).nl_last_error(handle)
        raise NlError(rc, msg.decode() if msg else "")
