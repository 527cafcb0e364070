from . import bebuzen, kekevik, lizezen, minicpm4, moputar, patadra, pugavik  # noqa: F401
