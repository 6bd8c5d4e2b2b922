// Causal attention over EVERY earlier key on ragged batches, bf16 MFMA (gfx950 only): the lean path of latent_attn.hip (no window, chunk, pooled rows or cap), and
// differential attention -- two maps per head over the same values, joined in the same kernel.
//
// A workgroup is four waves.  With one map, wave w owns query rows 32 w .. + 31 of a 128-row tile; with two maps the tile is 64 rows and waves 0, 1 run map 1,
// waves 2, 3 map 2 of the same rows: keys of both maps lie side by side in LDS, the value tile is staged once for both.  Scores are computed transposed,
// S^T = K Q^T (v_mfma_f32_32x32x16_bf16: A = 32 keys x 16 features from LDS, B = the lane's own query), so a lane holds 16 of every 32 keys of ONE query; softmax
// statistics and the rescale factor of O^T = V^T P^T are lane-local plus one exchange with lane ^ 32, and P is the B operand of that product as it stands in
// registers.  The value tile is row-major in LDS; its transposed fragments come from the LDS transpose read, whose key order inside a 16-key block -- rows
// 4 hf + 0..3, then 8 + 4 hf + 0..3 -- is the order in which the lane holds its scores.
// The next tile's keys and values are (but for the widest rows) requested before the current tile's arithmetic; only steps that reach a row's own position are masked; tiles with the
// most keys start first.  Options: a sink in the denominator, or sigmoid weights instead of the softmax (SIG); key splits as in latent_attn.hip.
#include "latent_attn.h"

#define ST(s) ((hipStream_t)(s))
#define LOG2E 1.4426950408889634f

struct DiffJoinArgs {  // the join of two maps: o = a1 - lam a2, o / sqrt(mean(o^2) + eps) * c, times sigmoid(gate) element by element
    const float* gate;  // fp32 rows [H x DV] or NULL
    int64_t ldg;
    float lam, eps, c;
};

template <int DKS, int NVB, bool SIG, int MAPS>
__global__ __launch_bounds__(256, NVB <= 4 && DKS * MAPS <= 16 ? 2 : 1) void latent_attn_full_kernel(LatAttnArgs p, DiffJoinArgs dj) {
    constexpr int DKP = DKS * 16, KROW = MAPS * DKP, DVP = NVB * 32, KLD = KROW + 8, VLD = DVP == 32 ? 32 : DVP + 32;
    constexpr int NKU = KROW / 32, NVU = NVB;         // 16-byte words of the key / value tile per thread: 64 * KROW / 8 / 256 and 64 * DVP / 8 / 256
    constexpr bool AHEAD = NVB < 8 || KROW <= 160;    // request the next tile during the current one's arithmetic, unless the widest rows leave no registers for it
    constexpr int ROWS = LAT_MQ / MAPS, JLD = DVP + 4;  // rows of a tile; row pitch of the exchange buffer of the join
    constexpr int SM_KV = 64 * (KLD + VLD) * 2, SM_J = MAPS == 2 ? ROWS * JLD * 4 : 0;
    __shared__ __attribute__((aligned(16))) unsigned char smem[SM_KV > SM_J ? SM_KV : SM_J];
    bf16_t* Ks = (bf16_t*)smem;
    bf16_t* Vs = Ks + 64 * KLD;
    const int s = blockIdx.z, tm = ROWS / p.hm;
    const int tiles = gridDim.x / p.splits;
    const int tile = tiles - 1 - (int)(blockIdx.x / p.splits), split = blockIdx.x % p.splits;
    const int tok0 = tile * tm, head0 = blockIdx.y * p.hm;
    const int n_new = p.n_new[s], past = p.past[s];
    if (tok0 >= n_new) return;
    const int64_t qr0 = p.q_row0[s], k1r0 = p.k1_row0[s], k2r0 = p.k2_row0[s], vr0 = p.v_row0[s];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ln = lane & 31, hf = lane >> 5;
    const int map = MAPS == 2 ? wave >> 1 : 0;
    const int DK = p.D1 + p.D2;
    const int kvh = head0 / p.kv_rep;
    const bf16_t* K1 = (const bf16_t*)p.K1 + k1r0 * p.ldk1 + (int64_t)kvh * p.k1_hs;
    const bf16_t* K2 = (const bf16_t*)p.K2 + k2r0 * p.ldk2;
    const bf16_t* V = (const bf16_t*)p.V + vr0 * p.ldv + (int64_t)kvh * p.v_hs;
    // this lane's query
    const int row = MAPS == 2 ? 32 * (wave & 1) + ln : 32 * wave + ln;
    const int tok = tok0 + row / p.hm, head = head0 + row % p.hm;
    const bool row_ok = tok < n_new && head < p.H;
    const int lim = row_ok ? past + tok : -1;
    bf16x8 qf[DKS];
    {
        const float* qrow = p.Q + (qr0 + (row_ok ? tok : 0)) * p.ldq + (int64_t)(row_ok ? head : 0) * p.q_hs + (MAPS == 2 ? map * p.D1 : 0);
#pragma unroll
        for (int st = 0; st < DKS; ++st) {
            float v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int d = 16 * st + 8 * hf + j;
                v[j] = (row_ok && d < DK) ? qrow[d] : 0.f;
            }
            const u32x4 pk = {pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]), pack_bf2(v[4], v[5]), pack_bf2(v[6], v[7])};
            qf[st] = __builtin_bit_cast(bf16x8, pk);
        }
    }
    const int n_keys = past + min(tok0 + tm, n_new);
    const int all_steps = (n_keys + 63) / 64;
    int v_lo = 0, v_hi = all_steps;
    if (p.splits > 1) {
        const int per = (all_steps + p.splits - 1) / p.splits;
        v_lo = min(all_steps, split * per);
        v_hi = min(all_steps, v_lo + per);
    }
    // the last key any row of this wave sees, and the last one that all of its rows see
    int wave_lim = lim, wave_all = row_ok ? lim : 0x7fffffff;
#pragma unroll
    for (int of = 32; of > 0; of >>= 1) wave_lim = max(wave_lim, __shfl_xor(wave_lim, of, 64)), wave_all = min(wave_all, __shfl_xor(wave_all, of, 64));
    wave_lim = __builtin_amdgcn_readfirstlane(wave_lim);
    wave_all = __builtin_amdgcn_readfirstlane(wave_all);

    f32x16 oacc[NVB];
#pragma unroll
    for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
        for (int i = 0; i < 16; ++i) oacc[vb][i] = 0.f;
    const float NEG = -__builtin_huge_valf();
    float m_run = NEG, l_run = 0.f;  // m_run in units of the raw dot product
    const float sc2 = p.scale * LOG2E;
    const float sgb = SIG ? p.sig_bias[row_ok ? head : 0] * LOG2E : 0.f;

    const u32x4 zero4 = {0u, 0u, 0u, 0u};
    u32x4 kreg[NKU], vreg[NVU];
    auto fetch = [&](int j0) {
#pragma unroll
        for (int u = 0; u < NKU; ++u) {
            const int c = tid + 256 * u, key = c / (KROW / 8), d0 = (c % (KROW / 8)) * 8, j = j0 + key;
            const int m = MAPS == 2 ? d0 / DKP : 0, d = MAPS == 2 ? d0 % DKP : d0;
            kreg[u] = zero4;
            if (j < n_keys && d < DK) kreg[u] = d < p.D1 ? *(const u32x4*)(K1 + (int64_t)j * p.ldk1 + m * p.D1 + d) : *(const u32x4*)(K2 + (int64_t)j * p.ldk2 + (d - p.D1));
        }
#pragma unroll
        for (int u = 0; u < NVU; ++u) {
            const int c = tid + 256 * u, key = c / (DVP / 8), d = (c % (DVP / 8)) * 8, j = j0 + key;
            vreg[u] = zero4;
            if (j < n_keys && d < p.DV) vreg[u] = *(const u32x4*)(V + (int64_t)j * p.ldv + d);
        }
    };
    auto stash = [&]() {
#pragma unroll
        for (int u = 0; u < NKU; ++u) {
            const int c = tid + 256 * u;
            *(u32x4*)&Ks[(c / (KROW / 8)) * KLD + (c % (KROW / 8)) * 8] = kreg[u];
        }
#pragma unroll
        for (int u = 0; u < NVU; ++u) {
            const int c = tid + 256 * u;
            *(u32x4*)&Vs[(c / (DVP / 8)) * VLD + (c % (DVP / 8)) * 8] = vreg[u];
        }
    };
    // transpose reads of the value tile: lane l addresses row 4 (l >> 5) + ((l >> 2) & 3), four columns at 16 ((l >> 4) & 1) + 4 (l & 3)
    const bf16_t* vtr = Vs + (4 * hf + ((lane >> 2) & 3)) * VLD + 16 * ((lane >> 4) & 1) + 4 * (lane & 3);
    typedef __attribute__((address_space(3))) bf16x4* lds4_t;

    if (AHEAD && v_lo < v_hi) fetch(v_lo * 64);
    for (int v = v_lo; v < v_hi; ++v) {
        const int j0 = v * 64;
        if (!AHEAD) fetch(j0);
        __syncthreads();  // the previous tile is consumed
        stash();
        __syncthreads();
        if (AHEAD && v + 1 < v_hi) fetch(j0 + 64);
        if (j0 > wave_lim) continue;  // every key of this step lies behind the wave's rows (the barriers are still reached by all)
        f32x16 sacc[2];
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
            for (int i = 0; i < 16; ++i) sacc[kb][i] = 0.f;
#pragma unroll
        for (int st = 0; st < DKS; ++st)
#pragma unroll
            for (int kb = 0; kb < 2; ++kb) {
                const bf16x8 a = *(const bf16x8*)&Ks[(kb * 32 + ln) * KLD + map * DKP + 16 * st + 8 * hf];
                sacc[kb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, qf[st], sacc[kb], 0, 0, 0);
            }
        // ---- weights of the lane's query (keys kb * 32 + 8 g + 4 hf + i)
        if (j0 + 63 > wave_all) {  // wave-uniform: only steps that reach a row's own position hide keys
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int r = 0; r < 16; ++r)
                    if (j0 + kb * 32 + 8 * (r >> 2) + 4 * hf + (r & 3) > lim) sacc[kb][r] = NEG;
        }
        if constexpr (SIG) {
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int r = 0; r < 16; ++r)  // a hidden key's -inf gives 0
                    sacc[kb][r] = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-fmaf(sacc[kb][r], sc2, sgb)));
        } else {
            float mx = NEG;
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sacc[kb][r]);
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            const float m_new = fmaxf(m_run, mx);
            const float base = m_new == NEG ? 0.f : m_new * sc2;
            const float f = m_new == m_run ? 1.0f : __builtin_amdgcn_exp2f(fmaf(m_run, sc2, -base));
            float sum = 0.f;
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    const float e = __builtin_amdgcn_exp2f(fmaf(sacc[kb][r], sc2, -base));
                    sacc[kb][r] = e;
                    sum += e;
                }
            sum += __shfl_xor(sum, 32, 64);
            l_run = l_run * f + sum;
            m_run = m_new;
            if (!__all(f == 1.0f)) {
#pragma unroll
                for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
                    for (int i = 0; i < 16; ++i) oacc[vb][i] *= f;
            }
        }
        // ---- O^T += V^T P^T, 16 keys at a time
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            const int kb = t >> 1, g = 8 * (t & 1);
            const u32x4 pk = {pack_bf2(sacc[kb][g + 0], sacc[kb][g + 1]), pack_bf2(sacc[kb][g + 2], sacc[kb][g + 3]), pack_bf2(sacc[kb][g + 4], sacc[kb][g + 5]),
                              pack_bf2(sacc[kb][g + 6], sacc[kb][g + 7])};
            const bf16x8 pf = __builtin_bit_cast(bf16x8, pk);
#pragma unroll
            for (int vb = 0; vb < NVB; ++vb) {
                const bf16_t* at = vtr + 16 * t * VLD + 32 * vb;
                const bf16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4_t)(at)), hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4_t)(at + 8 * VLD));
                const bf16x8 a = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
                oacc[vb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pf, oacc[vb], 0, 0, 0);
            }
        }
    }
    if (p.splits > 1) {  // partial results (maxima in base-2 units); rows that see nothing keep max = -inf and sum = 0; two maps: rows 64 .. 127 are map 2
        const int64_t blk = (((int64_t)s * gridDim.y + blockIdx.y) * tiles + tile) * p.splits + split;
        float* base = p.ws + blk * (int64_t)(LAT_MQ * (2 + DVP));
        const int wrow = 32 * wave + ln;
        if (hf == 0) base[wrow] = m_run * sc2, base[LAT_MQ + wrow] = l_run;
#pragma unroll
        for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
            for (int g = 0; g < 4; ++g)
                *(f32x4*)(base + 2 * LAT_MQ + (int64_t)wrow * DVP + vb * 32 + 8 * g + 4 * hf) = f32x4{oacc[vb][4 * g], oacc[vb][4 * g + 1], oacc[vb][4 * g + 2], oacc[vb][4 * g + 3]};
        return;
    }
    float inv = SIG ? 1.0f : 1.0f / l_run;
    if (!SIG && p.sink && row_ok) {  // the sink joins the denominator (statistics in base-2 units)
        const float sk = p.sink[head] * LOG2E, mr = m_run * sc2, m2 = fmaxf(mr, sk), f = exp2f(mr - m2);
        inv = f / (l_run * f + exp2f(sk - m2));
    }
    if constexpr (MAPS == 2) {
        float* J = (float*)smem;
        __syncthreads();  // every wave has left the loop: the tiles' memory is free
        if (map == 1) {
#pragma unroll
            for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
                for (int g = 0; g < 4; ++g)
                    *(f32x4*)&J[row * JLD + vb * 32 + 8 * g + 4 * hf] = f32x4{oacc[vb][4 * g], oacc[vb][4 * g + 1], oacc[vb][4 * g + 2], oacc[vb][4 * g + 3]} * inv;
        }
        __syncthreads();
        if (map == 1) return;
        float ssq = 0.f;
#pragma unroll
        for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const f32x4 a2 = *(const f32x4*)&J[row * JLD + vb * 32 + 8 * g + 4 * hf];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float o = oacc[vb][4 * g + i] * inv - dj.lam * a2[i];
                    oacc[vb][4 * g + i] = o;
                    ssq += o * o;
                }
            }
        ssq += __shfl_xor(ssq, 32, 64);  // columns beyond DV are zero in both maps
        inv = dj.c / sqrtf(ssq / (float)p.DV + dj.eps);
    }
    if (!row_ok) return;
    const int64_t o0 = (qr0 + tok) * p.ldo + (int64_t)head * p.o_hs;
    const float* gate = MAPS == 2 && dj.gate ? dj.gate + (qr0 + tok) * dj.ldg + (int64_t)head * p.DV : nullptr;
#pragma unroll
    for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
            const int dv = vb * 32 + 8 * g + 4 * hf;
            if (dv >= p.DV) continue;
            f32x4 v = f32x4{oacc[vb][4 * g], oacc[vb][4 * g + 1], oacc[vb][4 * g + 2], oacc[vb][4 * g + 3]} * inv;
            if (gate) {
                const f32x4 gq = *(const f32x4*)(gate + dv);
#pragma unroll
                for (int i = 0; i < 4; ++i) v[i] *= gate_of(gq[i]);
            }
            if (p.o_dt == MI355_DT_F32) *(f32x4*)((float*)p.O + o0 + dv) = v;
            else *(u32x2*)((bf16_t*)p.O + o0 + dv) = u32x2{pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3])};
        }
}

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
    if (dj.gate) {
        const f32x4 g = *(const f32x4*)(dj.gate + t * dj.ldg + (int64_t)head * p.DV + dv);
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] *= gate_of(g[i]);
    }
    *(u32x2*)((bf16_t*)p.O + t * p.ldo + (int64_t)head * p.o_hs + dv) = u32x2{pack_bf2(o[0], o[1]), pack_bf2(o[2], o[3])};
}

template <int DKS, bool SIG, int MAPS>
static void launch_full(const LatAttnArgs& p, const DiffJoinArgs& dj, dim3 grid, hipStream_t st) {
    if (p.DV <= 32) latent_attn_full_kernel<DKS, 1, SIG, MAPS><<<grid, 256, 0, st>>>(p, dj);
    else if (p.DV <= 64) latent_attn_full_kernel<DKS, 2, SIG, MAPS><<<grid, 256, 0, st>>>(p, dj);
    else if (p.DV <= 128) latent_attn_full_kernel<DKS, 4, SIG, MAPS><<<grid, 256, 0, st>>>(p, dj);
    else latent_attn_full_kernel<DKS, 8, SIG, MAPS><<<grid, 256, 0, st>>>(p, dj);
}

bool latent_attn_full_launch(const LatAttnArgs& p, dim3 grid, hipStream_t st) {
    const int DK = p.D1 + p.D2;
    const DiffJoinArgs none = {nullptr, 0, 0.f, 0.f, 0.f};
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
    p.scale = scale, p.kv_rep = kv_rep, p.splits = 1;
    const DiffJoinArgs dj = {gate, ldg, lam, eps, c};
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
