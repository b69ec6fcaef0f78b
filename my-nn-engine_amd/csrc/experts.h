// Sparse feed-forward (experts.hip): a token goes through the `top` experts with the largest scores sigmoid(W_router x), each
// over the input times its score: sum of W_down(silu(s W_gate x) * (s W_up x)).
#pragma once
#include "dense.h"

namespace mynn {

struct ExpertParams {
    int E, top, ld, fp;       // experts, experts per token, padded width and feed-forward
    const void *gu, *down;    // T [E][2 fp, ld] (gate and up rows interleaved in groups of 32), [E][ld, fp]
    // one row
    const float *x;           // the row, f32
    const float *logits;      // [E]
    void *hmid;               // T [top, fp]
    int32_t *chosen;          // [top]
    // several rows
    int rows;
    const void *router;       // T [E, ld]
    const void *act;          // T [rows, ld]
    int32_t *choice;          // [rows, top]
    float *score;             // [rows, top]
    // (assignment = row * top + i) sorted by expert, every expert's share padded to whole tiles
    int32_t *tile_expert;     // [max_tiles], -1: not used
    int32_t *slot;            // [max_tiles * rows of a tile] assignment, -1: padding
    void *hsort;              // T [max_tiles * rows of a tile, fp]
    float *parts;             // f32 [rows * top, ld] (top > 1)
    void *y;                  // T [rows, ld]
};
// rows of a tile: large ones once the experts have enough rows to fill them; tiles that any split of the rows needs
inline int expert_group_rows(int rows, int E, int top) { return (long)rows * top >= 192L * E ? 256 : 128; }
inline int expert_tiles(int rows, int E, int top, int group_rows) {
    const long a = (long)rows * top;
    return (int)(a / group_rows + (a < E ? a : E));
}
// one row: y = the experts' sum; x and the router's logits are there
int expert_gateup_row(const ExpertParams &p, int dtype, hipStream_t s);
int expert_down_row(const ExpertParams &p, int dtype, hipStream_t s);
bool expert_row_supported(int ld, int fp, int top);
// several rows: scores and choice from the f32 rows x [rows, ld]; the sorted order; the two products; the sum
int expert_route(const ExpertParams &p, int dtype, hipStream_t s);
int expert_sort(const ExpertParams &p, hipStream_t s);
int expert_gateup(const ExpertParams &p, int dtype, hipStream_t s);
int expert_down(const ExpertParams &p, int dtype, hipStream_t s);
int expert_sum(const ExpertParams &p, int dtype, hipStream_t s);

}  // namespace mynn
