from . import bebuzen, kekevik, minicpm4, moputar, patadra, pugavik  # noqa: F401
