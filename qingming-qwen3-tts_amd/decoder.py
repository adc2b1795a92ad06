"""ctypes binding of libqm_decoder.so: the decoder language models' engine and operators.  Mirrors include/qm_decoder.h.
Device pointers are raw addresses (or torch tensors in the operator helpers); the library itself never sees torch."""
import ctypes as C
import os

import numpy as np

HERE = os.path.dirname(os.path.abspath(__file__))
_LIB_PATH = os.path.join(HERE, "lib", "libqm_decoder.so")
_lib = None

_P, _I32, _I64, _U64, _F = C.c_void_p, C.c_int32, C.c_int64, C.c_uint64, C.c_float


def _structure(name, *fields):
    return type(name, (C.Structure,), {"_fields_": list(fields)})


def _same(kind, names):
    return [(n, kind) for n in names.split()]


ResidualTerm = _structure("ResidualTerm", *_same(_P, "y norm_w"), ("ld", _I64), ("scale", _F), ("reserved", _I32))
ResidualNorm = _structure("ResidualNorm", *_same(_P, "x_in embed tokens bigram row_map step_vec norm_w x_out h"), ("ld_h", _I64),
                          *_same(_I32, "width vocab terms"), ("eps", _F), *_same(_I32, "buckets mul_prev mul_cur reserved"),
                          ("term", ResidualTerm * 3))
GatedNorm = _structure("GatedNorm", *_same(_P, "o weight gate out"), *_same(_I64, "ld_o ld_gate ld_out"), *_same(_I32, "groups size"),
                       ("eps", _F), ("silu", _I32))
DecoderLinear = _structure("DecoderLinear", *_same(_P, "x w w_up out32 out"), *_same(_I64, "ldx ldo"), *_same(_I32, "n k"))
AttentionPartials = _structure("AttentionPartials", *_same(_P, "ml acc"), *_same(_I32, "heads vdim splits keys_per_split"))
ChunkAttention = _structure("ChunkAttention", *_same(_P, "proj frequency q_rot k_cache v_cache out"), ("part", AttentionPartials),
                            ("position_dev", _P), *_same(_I64, "ld_proj ld_out"), *_same(_I32, "position rows"),
                            *_same(_I32, "heads kv_heads dim vdim k_stride v_stride ring chunk rot_dims k_column v_column"), ("scale", _F), ("options", _I32), ("reserved", _I32))
DecayAttention = _structure("DecayAttention", *_same(_P, "proj powers state out scratch frequency position_dev"),
                            *_same(_I64, "ld_proj scratch_floats"), *_same(_I32, "rows heads dim vdim q_column k_column v_column options rot_dims position"),
                            ("k_scale", _F), ("reserved", _I32))
GeneralDelta = _structure("GeneralDelta", *_same(_P, "proj w2 w0 a_bias state out scratch"), *_same(_I64, "ld_proj scratch_floats"),
                          *_same(_I32, "rows heads dim rank r_column k_column v_column a_column z_column"), ("unit_eps", _F))
LatentRows = _structure("LatentRows", *_same(_P, "proj q_norm kv_norm frequency position_dev q_latent latent_cache key_cache"),
                        *_same(_I64, "ld_proj ld_q ld_latent"), *_same(_I32, "position rows q_rank kv_rank rot_dim key_stride q_column kv_column"),
                        *_same(_F, "eps magnitude"))
LatentAttention = _structure("LatentAttention", *_same(_P, "q frequency up_k up_v latent_cache key_cache out q_scratch ml acc expanded position_dev"),
                             *_same(_I64, "ld_query ld_latent ld_out expanded_bytes"),
                             *_same(_I32, "position rows heads dim rot_dim vdim kv_rank key_stride splits up_rows up_v_row options"),
                             *_same(_F, "scale magnitude"))
Experts = _structure("Experts", *_same(_P, "x logits gate up down out32 scratch"), *_same(_I64, "ld_logits scratch_bytes"),
                     *_same(_I32, "rows experts top width_p ff_p options"))
DECAY_POWERS = 65
DECAY_ROTARY = ATTENTION_ROWS = EXPERTS_ROWS = 1

_SIGNATURES = {
    "qm_residual_norm_rows": (_I32, [C.POINTER(ResidualNorm), _I32, _I32, _P]),
    "qm_gated_norm_rows": (_I32, [C.POINTER(GatedNorm), _I32, _I32, _P]),
    "qm_decoder_linear_rows": (_I32, [C.POINTER(DecoderLinear), _I32, _I32, _I32, _P]),
    "qm_chunk_attention_rows": (_I32, [C.POINTER(ChunkAttention), _I32, _P]),
    "qm_decay_attention_scratch_floats": (_I64, [_I32, _I32, _I32, _I32]),
    "qm_decay_attention_rows": (_I32, [C.POINTER(DecayAttention), _P]),
    "qm_general_delta_scratch_floats": (_I64, [_I32, _I32, _I32]),
    "qm_general_delta_rows": (_I32, [C.POINTER(GeneralDelta), _P]),
    "qm_latent_rows_norm": (_I32, [C.POINTER(LatentRows), _I32, _P]),
    "qm_latent_query_stride": (_I32, [_I32, _I32]),
    "qm_latent_expanded_bytes": (_I64, [_I32] * 6),
    "qm_latent_attention_rows": (_I32, [C.POINTER(LatentAttention), _I32, _P]),
    "qm_expert_scratch_bytes": (_I64, [_I32] * 6),
    "qm_expert_rows": (_I32, [C.POINTER(Experts), _I32, _P]),
    "qm_decoder_last_error": (C.c_char_p, []),
    "qm_decoder_architecture": (C.c_char_p, [_I32]),
    "qm_decoder_check_config": (_I32, [C.c_char_p]),
    "qm_decoder_create": (_I32, [C.c_char_p, _I32, _I32, _I32, _I32, _P, C.POINTER(_P)]),
    "qm_decoder_destroy": (None, [_P]),
    "qm_decoder_info": (_I32, [_P, C.POINTER(_I64)]),
    "qm_decoder_open": (_I32, [_P, C.POINTER(_I32)]),
    "qm_decoder_close": (_I32, [_P, _I32]),
    "qm_decoder_step": (_I32, [_P, _I32, _P, _I32, _P, _I32, _P, _P]),
    "qm_decoder_generate": (_I32, [_P, _I32, _P, _I32, _I32, _I32, _I32, _F, _U64, _P, C.POINTER(_I32)]),
    "qm_decoder_set_path": (_I32, [_P, _I32]),
    "qm_decoder_enqueue": (_I32, [_P, _I32, _P, _I32]),
    "qm_decoder_synchronize": (_I32, [_P]),
}
EXPORTS = tuple(_SIGNATURES)


class DecoderError(RuntimeError):
    def __init__(self, code, message):
        super().__init__(f"{message} (code {code})")
        self.code = code


def lib_path():
    return _LIB_PATH


def lib():
    """Loads the shared library (once).  Raises FileNotFoundError if it was not built."""
    global _lib
    if _lib is None:
        if not os.path.exists(_LIB_PATH):
            raise FileNotFoundError(f"{_LIB_PATH} is missing: build it with `python qingming-qwen3-tts_amd/build.py`")
        handle = C.CDLL(_LIB_PATH)
        for name, (restype, argtypes) in _SIGNATURES.items():
            fn = getattr(handle, name)
            fn.restype, fn.argtypes = restype, argtypes
        _lib = handle
    return _lib


def build_if_missing():
    """Builds the library (and nothing else) if it is not there; of several processes one builds."""
    if os.path.exists(_LIB_PATH):
        return
    import fcntl
    import importlib.util
    spec = importlib.util.spec_from_file_location("qm_build", os.path.join(HERE, "build.py"))
    build = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(build)
    os.makedirs(build.LIB_DIR, exist_ok=True)
    with open(os.path.join(build.LIB_DIR, ".lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not os.path.exists(_LIB_PATH):
            build.build_decoder(verbose=False)


def _check(code):
    if code != 0:
        raise DecoderError(code, lib().qm_decoder_last_error().decode("utf-8", "replace"))


def architectures():
    """The architecture names (config.json's 'architecture') that the registry serves."""
    names = []
    while (name := lib().qm_decoder_architecture(len(names))) is not None:
        names.append(name.decode())
    return names


def check_config(path):
    _check(lib().qm_decoder_check_config(os.fsencode(path)))


class Decoder:
    """qm_decoder: a model directory's weights, the live sequences' caches and states, step and generate."""

    def __init__(self, model_dir, capacity, float32=False, sequences=1, max_rows=0, stream=0):
        self._handle = _P()
        _check(lib().qm_decoder_create(os.fsencode(model_dir), int(float32), capacity, sequences, max_rows, stream or None,
                                       C.byref(self._handle)))
        info = (_I64 * 8)()
        _check(lib().qm_decoder_info(self._handle, info))
        (self.vocab, self.width, self.layers, self.runs, self.capacity, self.sequences, self.max_rows, self.sequence_bytes) = list(info)

    def close_model(self):
        if self._handle:
            lib().qm_decoder_destroy(self._handle)
            self._handle = _P()

    def __del__(self):
        self.close_model()

    def open(self):
        sequence = _I32()
        _check(lib().qm_decoder_open(self._handle, C.byref(sequence)))
        return sequence.value

    def close(self, sequence):
        _check(lib().qm_decoder_close(self._handle, sequence))

    def step(self, sequence, tokens, want=(), streams=False):
        """The sequence's next tokens; logits [len(want)][vocab] at the wanted places (and with `streams` the residual stream
        behind every layer run, [runs][tokens][width])."""
        tokens = np.ascontiguousarray(tokens, dtype=np.int32)
        want = np.ascontiguousarray(want, dtype=np.int32)
        logits = np.zeros((len(want), self.vocab), dtype=np.float32)
        taps = np.zeros((self.runs, len(tokens), self.width), dtype=np.float32) if streams else None
        _check(lib().qm_decoder_step(self._handle, sequence, tokens.ctypes.data, len(tokens), want.ctypes.data, len(want),
                                     logits.ctypes.data, taps.ctypes.data if streams else None))
        return (logits, taps) if streams else logits

    def generate(self, sequence, prompt, maximum, stop_token=-1, top_k=0, temperature=1.0, seed=0):
        """The tokens that follow `prompt` (top_k 0: greedy)."""
        prompt = np.ascontiguousarray(prompt, dtype=np.int32)
        out = np.zeros(maximum, dtype=np.int32)
        produced = _I32()
        _check(lib().qm_decoder_generate(self._handle, sequence, prompt.ctypes.data, len(prompt), maximum, stop_token, top_k,
                                         temperature, seed, out.ctypes.data, C.byref(produced)))
        return out[:produced.value].copy()

    def set_path(self, path):
        _check(lib().qm_decoder_set_path(self._handle, path))

    def enqueue(self, sequence, tokens):
        tokens = np.ascontiguousarray(tokens, dtype=np.int32)
        _check(lib().qm_decoder_enqueue(self._handle, sequence, tokens.ctypes.data, len(tokens)))

    def synchronize(self):
        _check(lib().qm_decoder_synchronize(self._handle))
