/* The wide-weight projection kernels over BF16 operands: linear_wide.hip compiled with the other element type (linear_elem.h). */
#define GD_LINEAR_BF16 1
#include "linear_wide.hip"
