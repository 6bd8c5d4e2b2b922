// Causal attention over EVERY earlier key on ragged batches, bf16 MFMA (gfx950 only): the lean path of latent_attn.hip without window, chunk, pooled rows or cap, and
// differential attention -- two maps per head over the same values, joined in the same kernel.
#include "latent_attn_full.h"

#define ST(s) ((hipStream_t)(s))

// Joins the partial results of both maps' key splits: one wave per query row, four values per lane (DV <= 256).
__global__ __launch_bounds__(256) void diff_attn_combine_kernel(LatAttnArgs p, DiffJoinArgs dj, int DVP, int tiles, int gy, int n_seq) {
    const int lane = threadIdx.x & 63, half = LAT_MQ / 2;
    const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);  // (sequence, head tile, token tile, row)
    const int row = (int)(item % half);
    int64_t rest = item / half;
    const int tile = (int)(rest % tiles);
    rest /= tiles;
    const int by = (int)(rest % gy), s = (int)(rest / gy);
    if (s >= n_seq) return;
    const int tm = half / p.hm, tok = tile * tm + row / p.hm, head = by * p.hm + row % p.hm;
    if (tok >= p.n_new[s] || head >= p.H) return;
    const float* ws = p.ws + (((int64_t)s * gy + by) * tiles + tile) * p.splits * (int64_t)(LAT_MQ * (2 + DVP));
    const int64_t stride = (int64_t)LAT_MQ * (2 + DVP);
    const int dv = 4 * lane;
    const bool ok = dv < p.DV;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < 2; ++m) {
        const int r = m * half + row;
        float mx = -__builtin_huge_valf(), l = 0.f;
        for (int i = 0; i < p.splits; ++i) mx = fmaxf(mx, ws[i * stride + r]);
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int i = 0; i < p.splits; ++i) {
            const float mi = ws[i * stride + r];
            if (mi == -__builtin_huge_valf()) continue;
            const float f = exp2f(mi - mx);
            l += ws[i * stride + LAT_MQ + r] * f;
            if (ok) acc += f * *(const f32x4*)(ws + i * stride + 2 * LAT_MQ + (int64_t)r * DVP + dv);
        }
        o += (m == 0 ? 1.0f : -dj.lam) / l * acc;
    }
    const float ssq = wave_sum((o[0] * o[0] + o[1] * o[1]) + (o[2] * o[2] + o[3] * o[3]));
    if (!ok) return;
    o *= dj.c / sqrtf(ssq / (float)p.DV + dj.eps);
    const int64_t t = (int64_t)p.q_row0[s] + tok;
    if (p.gate) {
        const f32x4 g = *(const f32x4*)(p.gate + t * p.ldg + (int64_t)head * p.DV + dv);
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] *= gate_of(g[i]);
    }
    *(u32x2*)((bf16_t*)p.O + t * p.ldo + (int64_t)head * p.o_hs + dv) = u32x2{pack_bf2(o[0], o[1]), pack_bf2(o[2], o[3])};
}

bool latent_attn_full_launch(const LatAttnArgs& p, dim3 grid, hipStream_t st) {
    const int DK = p.D1 + p.D2;
    const DiffJoinArgs none = {0.f, 0.f, 0.f};
    if (p.DV > 256) return false;
    if (p.sig_bias) {
        if (DK <= 64) launch_full<4, true, 1>(p, none, grid, st);
        else if (DK <= 128) launch_full<8, true, 1>(p, none, grid, st);
        else return false;
        return true;
    }
    if (DK <= 64) launch_full<4, false, 1>(p, none, grid, st);
    else if (DK <= 128) launch_full<8, false, 1>(p, none, grid, st);
    else if (DK <= 192) launch_full<12, false, 1>(p, none, grid, st);
    else if (DK <= 256) launch_full<16, false, 1>(p, none, grid, st);
    else if (DK <= 320) launch_full<20, false, 1>(p, none, grid, st);
    else return false;
    return true;
}

extern "C" int mi355_diff_attn(int n_seq, int max_new, int H, int hm, int D, int DV, const float* Q, int64_t ldq, const void* K, int64_t ldk, const void* V, int64_t ldv,
                               void* O, int64_t ldo, const int* q_row0, const int* n_new, const int* past, const int* k_row0, float scale, int kv_rep, int splits, float* ws,
                               int64_t ws_floats, float lam, float eps, float c, const float* gate, int64_t ldg, void* stream) {
    MI355_REQUIRE(n_seq > 0 && n_seq <= 65535 && max_new > 0 && H > 0 && D > 0 && D <= 128 && D % 8 == 0 && DV > 0 && DV <= 256 && DV % 8 == 0 && Q && K && V && O && scale > 0.f,
                  "diff_attn: bad arguments (maps <= 128, values <= 256 wide, multiples of 8; scale > 0)");
    MI355_REQUIRE(kv_rep >= 1 && H % kv_rep == 0 && hm >= 1 && hm <= 32 && 32 % hm == 0 && kv_rep % hm == 0, "diff_attn: bad head grouping");
    MI355_REQUIRE(q_row0 && n_new && past && k_row0, "diff_attn: sequence descriptors missing");
    const int G = H / kv_rep;
    MI355_REQUIRE(ldq >= (int64_t)2 * H * D && ldk >= (int64_t)2 * G * D && ldv >= (int64_t)G * DV && ldo >= (int64_t)H * DV && (!gate || ldg >= (int64_t)H * DV), "diff_attn: rows too short");
    MI355_REQUIRE(ldk % 8 == 0 && ldv % 8 == 0 && ldo % 4 == 0 && ldg % 4 == 0 && ((uintptr_t)K & 15) == 0 && ((uintptr_t)V & 15) == 0 && ((uintptr_t)O & 7) == 0 && ((uintptr_t)gate & 15) == 0,
                  "diff_attn: rows must be 16-byte aligned");
    LatAttnArgs p = {};
    p.Q = Q, p.K1 = K, p.V = V, p.O = O, p.ldq = ldq, p.ldk1 = ldk, p.ldv = ldv, p.ldo = ldo;
    p.q_hs = 2 * D, p.k1_hs = 2 * D, p.v_hs = DV, p.o_hs = DV, p.D1 = D, p.D2 = 0, p.DV = DV, p.H = H, p.hm = hm, p.dt = MI355_DT_BF16, p.o_dt = MI355_DT_BF16;
    p.q_row0 = q_row0, p.n_new = n_new, p.past = past, p.k1_row0 = k_row0, p.k2_row0 = k_row0, p.v_row0 = k_row0;
    p.scale = scale, p.kv_rep = kv_rep, p.splits = 1, p.gate = gate, p.ldg = ldg;
    const DiffJoinArgs dj = {lam, eps, c};
    const int tm = LAT_MQ / 2 / hm;
    const int64_t gx = ((int64_t)max_new + tm - 1) / tm, gy = H / hm;
    const int DVP = DV <= 32 ? 32 : DV <= 64 ? 64 : DV <= 128 ? 128 : 256;
    MI355_REQUIRE(gy <= 65535 && gx * (splits > 1 ? splits : 1) < ((int64_t)1 << 31), "diff_attn: grid too large");
    if (splits > 1) {
        MI355_REQUIRE(splits <= 64 && ws && ((uintptr_t)ws & 15) == 0 && ws_floats >= (int64_t)n_seq * gy * gx * splits * LAT_MQ * (2 + DVP), "diff_attn: key splits need a larger workspace");
        p.splits = splits, p.ws = ws;
    }
    dim3 grid((unsigned)(gx * p.splits), (unsigned)gy, n_seq);
    if (D <= 32) launch_full<2, false, 2>(p, dj, grid, ST(stream));
    else if (D <= 64) launch_full<4, false, 2>(p, dj, grid, ST(stream));
    else launch_full<8, false, 2>(p, dj, grid, ST(stream));
    MI355_LAUNCH_CHECK("diff_attn");
    if (p.splits > 1) {
        const int64_t items = (int64_t)n_seq * gy * gx * (LAT_MQ / 2);
        diff_attn_combine_kernel<<<(unsigned)((items + 3) / 4), 256, 0, ST(stream)>>>(p, dj, DVP, (int)gx, (int)gy, n_seq);
        MI355_LAUNCH_CHECK("diff_attn(combine)");
    }
    return 0;
}
