"""MI355X (gfx950) back end for rust-model-inference's quantized matrix products.

``synth``  seeded synthetic tensors of the benchmark shapes (numpy only)
``folder`` model folders: safetensors writer, synthetic Ruvenex and Vogizen models (numpy only)
``gguf``   minimal GGUF v3 writer / mmap reader (synthetic Qwen3 file)
``hip``    ctypes binding of librmi_hip.so, the C ABI of include/rmi_hip.h
``kernel`` mirror of the reference's Kernel / Layer interface over that ABI
``decode`` decoder sessions (Qwen3, Ruvenex, Vogizen) over the device-resident decode entry points
``models`` registry: the session class of a model file or folder
``replay`` token ids through a session, step by step, logits to files (bin/trace_run)
``loader`` mirror of GGUFLoader over the library's parser; file -> HBM uploads

``hip``, ``kernel``, ``decode``, ``models``, ``replay`` and ``loader`` load the compiled library on first use and raise if it
is missing; nothing here computes on the CPU.
"""
import importlib

from . import folder, gguf, synth  # noqa: F401

_LAZY = ("hip", "kernel", "decode", "loader", "models", "replay")


def __getattr__(name):
    if name in _LAZY:
        return importlib.import_module(f"{__name__}.{name}")
    if name == "init":
        return importlib.import_module(f"{__name__}.hip").init
    raise AttributeError(name)
