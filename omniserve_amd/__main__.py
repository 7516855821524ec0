"""python -m omniserve_amd: see omniserve_amd/cli.py."""
import sys

from .cli import main

sys.exit(main())
