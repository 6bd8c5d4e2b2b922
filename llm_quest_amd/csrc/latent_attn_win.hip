// Causal attention under a window (with kept first tokens) or a chunk, with capped scores or a distance bias, on ragged batches: the lean bf16 MFMA kernel of
// latent_attn_full.h with these options (gfx950 only).
#include "latent_attn_full.h"

bool latent_attn_win_launch(const LatAttnArgs& p, dim3 grid, hipStream_t st) {
    const int DK = p.D1 + p.D2;
    const DiffJoinArgs none = {0.f, 0.f, 0.f};
    if (p.DV > 256 || p.sig_bias) return false;
    if (p.softcap > 0.f || p.slope) {
        if (DK <= 64) launch_full<4, false, 1, LAT_SCORE>(p, none, grid, st);
        else if (DK <= 128) launch_full<8, false, 1, LAT_SCORE>(p, none, grid, st);
        else if (DK <= 192) launch_full<12, false, 1, LAT_SCORE>(p, none, grid, st);
        else if (DK <= 256) launch_full<16, false, 1, LAT_SCORE>(p, none, grid, st);
        else return false;
        return true;
    }
    if (DK <= 64) launch_full<4, false, 1, LAT_WINDOW>(p, none, grid, st);
    else if (DK <= 128) launch_full<8, false, 1, LAT_WINDOW>(p, none, grid, st);
    else if (DK <= 192) launch_full<12, false, 1, LAT_WINDOW>(p, none, grid, st);
    else if (DK <= 256) launch_full<16, false, 1, LAT_WINDOW>(p, none, grid, st);
    else return false;
    return true;
}
