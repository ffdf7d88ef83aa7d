"""The model registry: which session class serves which architecture, and opening a model by its path.

A GGUF file names its architecture in its metadata (src/core/loader.rs:379-461), a model folder in config.json.
"""
import json
import os

from . import hip

# architecture of a model folder -> name of its session class in ``decode``
FOLDER_SESSIONS = {"Ruvenex": "RuvenexSession", "Vogizen": "VogizenSession"}

DTYPES = {"bfloat16": hip.DTYPE_BF16, "float32": hip.DTYPE_F32}


def folder_architecture(path):
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f).get("architecture")


def session_class(architecture):
    from . import decode

    name = FOLDER_SESSIONS.get(architecture)
    if name is None:
        raise ValueError(f"no session for architecture {architecture!r} (known: {', '.join(sorted(FOLDER_SESSIONS))})")
    return getattr(decode, name)


def open_session(path, capacity, dtype="bfloat16"):
    """The session of the model at `path`: a folder by its config.json, a file as GGUF (whose dtype is its own)."""
    if os.path.isdir(path):
        return session_class(folder_architecture(path))(path, capacity, DTYPES[dtype])
    from . import decode, loader

    with loader.GGUFLoader.from_file(path) as g:
        return decode.Qwen3Session.from_gguf(g, capacity)
