/* 256 x 256 tiles over [N,K] weights of the many-row F16 projection kernel (linear_tile.hip). */
#define GD_LINEAR_TILE_PART 1
#include "linear_tile.hip"
