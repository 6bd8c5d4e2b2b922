// The lean attention kernel (bf16 MFMA, gfx950 only): compiled by latent_attn_full.hip (every key j <= i, one or two maps) and latent_attn_win.hip (windows, chunks,
// capped scores, distance biases).
//
// A workgroup is four waves.  With one map, wave w owns query rows 32 w .. + 31 of a 128-row tile; with two maps the tile is 64 rows and waves 0, 1 run map 1,
// waves 2, 3 map 2 of the same rows: keys of both maps lie side by side in LDS, the value tile is staged once for both.  Scores are computed transposed,
// S^T = K Q^T (v_mfma_f32_32x32x16_bf16: A = 32 keys x 16 features from LDS, B = the lane's own query), so a lane holds 16 of every 32 keys of ONE query; softmax
// statistics and the rescale factor of O^T = V^T P^T are lane-local plus one exchange with lane ^ 32, and P is the B operand of that product as it stands in
// registers.  The value tile is row-major in LDS; its transposed fragments come from the LDS transpose read, whose key order inside a 16-key block -- rows
// 4 hf + 0..3, then 8 + 4 hf + 0..3 -- is the order in which the lane holds its scores.
// The next tile's keys and values are (but for the widest rows) requested before the current tile's arithmetic; only steps with a key that some row of the wave does not
// see are masked; tiles with the most keys start first.  A tile walks the 64-key steps of key_steps (kept first tokens, then its window).  Options: a sink in the
// denominator, or sigmoid weights instead of the softmax (SIG); key splits as in latent_attn.hip; a sigmoid gate on the output.
#pragma once
#include "latent_attn.h"

#define LOG2E 1.4426950408889634f

struct DiffJoinArgs {  // the join of two maps: o = a1 - lam a2, o / sqrt(mean(o^2) + eps) * c
    float lam, eps, c;
};

// What hides keys besides causality, and what happens to a score before its weight.
enum { LAT_ALL = 0,     // every key j <= i, plain scores
       LAT_WINDOW = 1,  // window (with kept first tokens) or chunk, plain scores
       LAT_SCORE = 2 }; // window / chunk / neither, capped scores and / or a distance bias

template <int DKS, int NVB, bool SIG, int MAPS, int OPT>
__global__ __launch_bounds__(256, NVB <= 4 && DKS * MAPS <= 16 ? 2 : 1) void latent_attn_full_kernel(LatAttnArgs p, DiffJoinArgs dj) {
    constexpr int DKP = DKS * 16, KROW = MAPS * DKP, DVP = NVB * 32, KLD = KROW + 8, VLD = DVP == 32 ? 32 : DVP + 32;
    constexpr int NKU = KROW / 32, NVU = NVB;         // 16-byte words of the key / value tile per thread: 64 * KROW / 8 / 256 and 64 * DVP / 8 / 256
    static_assert(OPT == LAT_ALL || (!SIG && MAPS == 1), "windows, caps and distance biases go with one softmax map");
    // request the next tile during the current one's arithmetic, unless wide rows leave no registers for it
    constexpr bool AHEAD = NVB < 4 || (NVB == 4 && !(OPT == LAT_SCORE && DKS >= 12)) || (NVB == 8 && KROW <= 160);
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
    KeySteps ks = {0, 0, (n_keys + 63) / 64};
    if constexpr (OPT != LAT_ALL) ks = key_steps(past + tok0, n_keys, p.window, p.keep_first, p.chunk);
    const int all_steps = ks.n;
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

    // the first key of a row's window or chunk (it grows with the row's position, so the wave's first and last rows bound it)
    const int row_lo = OPT == LAT_ALL ? 0 : tile_key_floor(lim, p.window, p.chunk);
    const int wave_lo_min = OPT == LAT_ALL || wave_lim < 0 ? 0 : tile_key_floor(wave_all, p.window, p.chunk);
    const int wave_lo_max = OPT == LAT_ALL || wave_lim < 0 ? 0 : tile_key_floor(wave_lim, p.window, p.chunk);

    f32x16 oacc[NVB];
#pragma unroll
    for (int vb = 0; vb < NVB; ++vb)
#pragma unroll
        for (int i = 0; i < 16; ++i) oacc[vb][i] = 0.f;
    const float NEG = -__builtin_huge_valf();
    float m_run = NEG, l_run = 0.f;  // m_run in units of the raw dot product (LAT_SCORE: of the final score, base 2)
    const float sc = p.scale * LOG2E, sc2 = OPT == LAT_SCORE ? 1.0f : sc;
    const float cap2 = OPT == LAT_SCORE ? p.softcap * LOG2E : 0.f, cap_in = OPT == LAT_SCORE && p.softcap > 0.f ? 2.0f * sc / p.softcap : 0.f;
    const float sl2 = OPT == LAT_SCORE && p.slope ? p.slope[row_ok ? head : 0] * LOG2E : 0.f;
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

    if (AHEAD && v_lo < v_hi) fetch(ks.key(v_lo));
    for (int v = v_lo; v < v_hi; ++v) {
        const int j0 = ks.key(v);
        if (!AHEAD) fetch(j0);
        __syncthreads();  // the previous tile is consumed
        stash();
        __syncthreads();
        if (AHEAD && v + 1 < v_hi) fetch(ks.key(v + 1));
        if (j0 > wave_lim) continue;  // every key of this step lies behind the wave's rows (the barriers are still reached by all)
        if (OPT != LAT_ALL && j0 + 63 < wave_lo_min && j0 >= p.keep_first) continue;  // ... or before the windows of all of them
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
        if constexpr (OPT == LAT_SCORE) {
            if (p.softcap > 0.f) {  // cap * tanh(s / cap) = cap - 2 cap / (exp(2 s / cap) + 1)
#pragma unroll
                for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                    for (int r = 0; r < 16; ++r) sacc[kb][r] = fmaf(-2.0f * cap2, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(sacc[kb][r] * cap_in)), cap2);
            } else {
#pragma unroll
                for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                    for (int r = 0; r < 16; ++r) sacc[kb][r] *= sc;
            }
            if (p.slope) {
                const float d0 = sl2 * (float)(j0 + 4 * hf - lim);
#pragma unroll
                for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                    for (int r = 0; r < 16; ++r) sacc[kb][r] += fmaf(sl2, (float)(kb * 32 + 8 * (r >> 2) + (r & 3)), d0);
            }
        }
        if constexpr (OPT != LAT_ALL) {
            if (j0 + 63 > wave_all || (j0 < wave_lo_max && j0 + 63 >= p.keep_first)) {  // wave-uniform: some row does not see some key of this step
                const int over = lim - j0 - 4 * hf, under = row_lo - j0 - 4 * hf, kept = p.keep_first - j0 - 4 * hf;
#pragma unroll
                for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                    for (int r = 0; r < 16; ++r) {
                        const int o = kb * 32 + 8 * (r >> 2) + (r & 3);
                        if (o > over || (o < under && o >= kept)) sacc[kb][r] = NEG;
                    }
            }
        } else if (j0 + 63 > wave_all) {  // wave-uniform: only steps that reach a row's own position hide keys
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
    const float* gate = p.gate ? p.gate + (qr0 + tok) * p.ldg + (int64_t)head * p.DV : nullptr;
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

template <int DKS, bool SIG, int MAPS, int OPT = LAT_ALL>
static void launch_full(const LatAttnArgs& p, const DiffJoinArgs& dj, dim3 grid, hipStream_t st) {
    if (p.DV <= 32) latent_attn_full_kernel<DKS, 1, SIG, MAPS, OPT><<<grid, 256, 0, st>>>(p, dj);
    else if (p.DV <= 64) latent_attn_full_kernel<DKS, 2, SIG, MAPS, OPT><<<grid, 256, 0, st>>>(p, dj);
    else if (p.DV <= 128) latent_attn_full_kernel<DKS, 4, SIG, MAPS, OPT><<<grid, 256, 0, st>>>(p, dj);
    else latent_attn_full_kernel<DKS, 8, SIG, MAPS, OPT><<<grid, 256, 0, st>>>(p, dj);
}
