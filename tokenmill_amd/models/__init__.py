"""Architectures. Importing this package registers each of them under its config.json name."""
from tokenmill_amd.models import gaborax, kasovik, lusolix, luzevik, modinex, qwen2, sanazen  # noqa: F401
from tokenmill_amd.models.decoder import DecoderModel, LayerCall

__all__ = ["DecoderModel", "LayerCall"]
