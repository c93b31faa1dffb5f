"""Reading the config.json of native designs: sections with known keys."""
import warnings
from typing import Any, Dict


def take_section(section: Dict[str, Any], where: str, required, optional=()) -> Dict[str, Any]:
    """The section itself; a missing key is an error, one that this build does not know is reported."""
    missing = sorted(set(required) - set(section))
    if missing:
        raise ValueError(f"{where}: missing keys {missing}")
    unknown = sorted(set(section) - set(required) - set(optional))
    if unknown:
        warnings.warn(f"{where}: unknown keys {unknown} are ignored")
    return section
