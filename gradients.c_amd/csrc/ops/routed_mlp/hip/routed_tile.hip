/* Projections of many rows packed by expert, each expert with its own weights: the tile kernel of the projections
 * (linear_tile.hip) over BF16 operands with a work list of (expert, row) tiles, and its launcher. */
#define GD_LINEAR_BF16 1
#define GD_LINEAR_TILE_GROUPED 1
#include "../../linear/hip/linear_tile.hip"
