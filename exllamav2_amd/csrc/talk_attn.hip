// talk_attn.hip -- grouped-head softmax attention over a paged cache whose heads exchange their scores before the softmax, for
// gfx950, + its C ABI.
//
// For a position p of a sequence and the keys j it sees (0 <= p - j < window):
//     a_g,j = c tanh(q_g . k_j / c)  (q rotated and scaled; c = softcap, 0: none),    s_h,j = sum_g T[h, g] a_g,j  over ALL heads,
//     o_h = sum_j exp(s_h,j) v_j / (exp(sink_h) + sum_j exp(s_h,j))                   (sink nullable: no such term)
// Query head h reads key / value head h / (heads / kv_heads).  The cache holds rotated keys [pages, page, kv_heads, dim] and values
// [pages, page, kv_heads, vdim] (window_attn.hip: exl2_kv_rot_append_ex writes them).  Rows of a step are a flat list (row r = position
// row_pos[r] of sequence row_seq[r]); a row's result depends only on its own (sequence, position).  Scores, their exchange, the
// softmax and the sums are fp32.
#include "hw.h"
#include "errors.h"
#include <stdint.h>

template <typename T> DEV float ta_ld(const T* p);
template <> DEV float ta_ld<u16>(const u16* p) { return bf16_to_f32(*p); }
template <> DEV float ta_ld<float>(const float* p) { return *p; }
template <typename T> DEV void ta_st(T* p, float v);
template <> DEV void ta_st<u16>(u16* p, float v) { *p = f32_to_bf16(v); }
template <> DEV void ta_st<float>(float* p, float v) { *p = v; }
// 16 bytes of T as floats
template <typename T> struct TaVec;
template <> struct TaVec<u16>
{
    static constexpr int N = 8;
    static DEV void load(const u16* p, float* f)
    {
        const u32x4 v = *(const u32x4*)p;
        #pragma unroll
        for (int i = 0; i < 4; i++) { f[2 * i] = as_f32(v[i] << 16); f[2 * i + 1] = as_f32(v[i] & 0xffff0000u); }
    }
};
template <> struct TaVec<float>
{
    static constexpr int N = 4;
    static DEV void load(const float* p, float* f)
    {
        const f32x4 v = *(const f32x4*)p;
        #pragma unroll
        for (int i = 0; i < 4; i++) f[i] = v[i];
    }
};
template <typename T> DEV void ta_ld2(const T* p, float& a, float& b);
template <> DEV void ta_ld2<u16>(const u16* p, float& a, float& b) { const u32 v = *(const u32*)p; a = as_f32(v << 16); b = as_f32(v & 0xffff0000u); }
template <> DEV void ta_ld2<float>(const float* p, float& a, float& b) { const f32x2 v = *(const f32x2*)p; a = v[0]; b = v[1]; }

// the wave's lanes meet around a tile of LDS that only they share: neither the hardware nor the compiler (whose alias analysis sees one
// lane's own addresses only) moves LDS accesses across it
DEV void ta_wave_lds() { wave_sync(); wait_lds_reads(); }

#define TA_NEG_BIG (-1.0e30f)
#define TA_KEYS 64                           // keys per step of the row kernel
#define TA_MAX_SPLIT 64

struct TalkArgs
{
    const void* q;                           // [rows, H, dim] rotated, scaled
    const void* k_cache; const void* v_cache;
    const float* talk;                       // [H, H]
    const float* sink;                       // [H] (nullable)
    const int* row_seq; const int* row_pos; const int* block_table; int bt_stride, page, page_shift;
    void* out;                               // [rows, H, vdim]
    int H, G, dim, vdim, window; float softcap;
    const int* row_list;                     // row kernel: the rows (nullable: 0, 1, ..)
    const int* tile_row0; const int* tile_rows;      // tile kernel: runs of <= 16 consecutive positions of one sequence
    // nsplit > 1 (row kernel): the key steps are dealt to nsplit workgroups; part_o fp32 [rows, H, nsplit, vdim] (sums relative to the
    // partial maximum), part_ml fp32 [rows, H, nsplit, 2] (maximum, sum)
    float* part_o; float* part_ml; int nsplit;
};

DEV float ta_soft_cap(float s, float cap) { return cap > 0.0f ? cap * tanhf(s / cap) : s; }
DEV long long ta_cache_row(const TalkArgs& a, const int* bt, int j)
{
    const int pg = a.page_shift >= 0 ? j >> a.page_shift : j / a.page;
    const int in = a.page_shift >= 0 ? j & (a.page - 1) : j % a.page;
    return (long long)bt[pg] * a.page + in;
}

// ---- one row per workgroup (decoded tokens; every shape and dtype) ---------------------------------------------------------------
// Keys go by TA_KEYS at a time: (kv head, up to four of its query heads, key) tasks make the capped scores, (head, key) tasks mix
// them over all heads, a wave per head joins the step to the head's running softmax, and (kv head, up to four of its query heads,
// pair of values) tasks add the step's weighted values to sums kept in LDS.

// q [H, dim], o [H, vdim] (both rounded up to whole 16-byte pieces), scores a and mixed s [H, TA_KEYS], running maximum / sum / correction [H]
HD size_t ta_row_smem(int H, int dim, int vdim)
{
    return sizeof(float) * ((size_t)((H * dim + 3) & ~3) + ((H * vdim + 3) & ~3) + 2 * (size_t)H * TA_KEYS + 3 * (size_t)H);
}

template <typename T, bool VEC>
KERNEL void __launch_bounds__(256) talk_attn_row_kernel(const TalkArgs a)
{
    DYN_SMEM(smem);
    SHARED long long krow[TA_KEYS];
    const int H = a.H, G = a.G, dim = a.dim, vd = a.vdim, hpg = H / G, quads = (hpg + 3) / 4;
    float* s_q = (float*)smem;
    float* s_o = s_q + ((H * dim + 3) & ~3);
    float* s_a = s_o + ((H * vd + 3) & ~3);
    float* s_p = s_a + H * TA_KEYS;
    float* s_m = s_p + H * TA_KEYS;
    float* s_l = s_m + H;
    float* s_c = s_l + H;
    const int t = tid(), lane = lane_id(), wv = wave_id();
    const int r = a.row_list ? a.row_list[bid_x()] : bid_x();
    const int split = bid_y();
    const int pos = a.row_pos[r];
    const int* bt = a.block_table + (long long)a.row_seq[r] * a.bt_stride;
    const int j_lo = max(0, pos - a.window + 1);
    const int total = pos - j_lo + 1;
    const int all_steps = (total + TA_KEYS - 1) / TA_KEYS;
    const int per_split = (all_steps + a.nsplit - 1) / a.nsplit;
    const int step0 = split * per_split, step1 = min(all_steps, step0 + per_split);
    const T* qr = (const T*)a.q + (long long)r * H * dim;
    for (int i = t; i < H * dim; i += 256) s_q[i] = ta_ld<T>(qr + i);
    for (int i = t; i < H * vd; i += 256) s_o[i] = 0.0f;
    const bool with_sink = a.sink && split == 0;                 // the sink counts once
    for (int i = t; i < H; i += 256) { s_m[i] = with_sink ? a.sink[i] : TA_NEG_BIG; s_l[i] = with_sink ? 1.0f : 0.0f; }
    for (int step = step0; step < step1; step++)
    {
        const int k0 = step * TA_KEYS, nc = min(TA_KEYS, total - k0);
        if (t < TA_KEYS) krow[t] = ta_cache_row(a, bt, j_lo + k0 + min(t, nc - 1));
        block_sync();
        for (int i = t; i < G * quads * TA_KEYS; i += 256)
        {
            const int key = i % TA_KEYS, gq = i / TA_KEYS, g = gq / quads, h0 = g * hpg + (gq % quads) * 4, nh = min(4, g * hpg + hpg - h0);
            const T* kr = (const T*)a.k_cache + (krow[key] * G + g) * dim;
            float d[4] = {0.0f, 0.0f, 0.0f, 0.0f};
            if (VEC)
            {
                constexpr int N = TaVec<T>::N;
                #pragma unroll 4
                for (int e = 0; e < dim; e += N)
                {
                    float kv[N];
                    TaVec<T>::load(kr + e, kv);
                    #pragma unroll
                    for (int n = 0; n < 4; n++)
                    {
                        const float* qh = s_q + (h0 + min(n, nh - 1)) * dim + e;
                        #pragma unroll
                        for (int x = 0; x < N; x++) d[n] = fmaf(qh[x], kv[x], d[n]);
                    }
                }
            }
            else
                for (int e = 0; e < dim; e++)
                {
                    const float kv = ta_ld<T>(kr + e);
                    #pragma unroll
                    for (int n = 0; n < 4; n++) d[n] = fmaf(s_q[(h0 + min(n, nh - 1)) * dim + e], kv, d[n]);
                }
            #pragma unroll
            for (int n = 0; n < 4; n++)
                if (n < nh) s_a[(h0 + n) * TA_KEYS + key] = ta_soft_cap(d[n], a.softcap);
        }
        block_sync();
        for (int i = t; i < H * TA_KEYS; i += 256)
        {
            const int key = i % TA_KEYS, h = i / TA_KEYS;
            const float* tr = a.talk + h * H;
            float s = 0.0f;
            for (int g = 0; g < H; g++) s = fmaf(tr[g], s_a[g * TA_KEYS + key], s);
            s_p[i] = key < nc ? s : TA_NEG_BIG;
        }
        block_sync();
        for (int h = wv; h < H; h += 4)
        {
            const float s = s_p[h * TA_KEYS + lane];
            const float m0 = s_m[h], m1 = fmaxf(m0, wave_allreduce_max(s));
            const float p = lane < nc ? expf(s - m1) : 0.0f;
            const float ps = wave_allreduce_add(p);
            s_p[h * TA_KEYS + lane] = p;
            if (lane == 0)
            {
                const float c = expf(m0 - m1);
                s_c[h] = c; s_m[h] = m1; s_l[h] = s_l[h] * c + ps;
            }
        }
        block_sync();
        const int vw = VEC ? 2 : 1;
        for (int i = t; i < G * quads * (vd / vw); i += 256)
        {
            const int e = (i % (vd / vw)) * vw, gq = i / (vd / vw), g = gq / quads, h0 = g * hpg + (gq % quads) * 4, nh = min(4, g * hpg + hpg - h0);
            float o0[4], o1[4];
            #pragma unroll
            for (int n = 0; n < 4; n++)
            {
                const int h = h0 + min(n, nh - 1);
                o0[n] = s_o[h * vd + e] * s_c[h];
                o1[n] = VEC ? s_o[h * vd + e + 1] * s_c[h] : 0.0f;
            }
            #pragma unroll 8
            for (int key = 0; key < nc; key++)
            {
                const T* vr = (const T*)a.v_cache + (krow[key] * G + g) * vd + e;
                float v0, v1 = 0.0f;
                if (VEC) ta_ld2<T>(vr, v0, v1); else v0 = ta_ld<T>(vr);
                #pragma unroll
                for (int n = 0; n < 4; n++)
                {
                    const float p = s_p[(h0 + min(n, nh - 1)) * TA_KEYS + key];
                    o0[n] = fmaf(p, v0, o0[n]);
                    if (VEC) o1[n] = fmaf(p, v1, o1[n]);
                }
            }
            #pragma unroll
            for (int n = 0; n < 4; n++)
                if (n < nh) { s_o[(h0 + n) * vd + e] = o0[n]; if (VEC) s_o[(h0 + n) * vd + e + 1] = o1[n]; }
        }
        block_sync();                                            // krow and the probabilities are rewritten by the next step
    }
    block_sync();
    for (int i = t; i < H * vd; i += 256)
    {
        const int h = i / vd;
        if (a.nsplit == 1) { ta_st<T>((T*)a.out + (long long)r * H * vd + i, s_l[h] > 0.0f ? s_o[i] / s_l[h] : 0.0f); continue; }
        const long long pi = ((long long)r * H + h) * a.nsplit + split;
        a.part_o[pi * vd + i % vd] = s_o[i];
        if (i % vd == 0) { a.part_ml[pi * 2] = s_m[h]; a.part_ml[pi * 2 + 1] = s_l[h]; }
    }
}

// grid (rows, heads): joins the nsplit partial results of a row's head
template <typename T>
KERNEL void __launch_bounds__(64) talk_attn_merge_kernel(const TalkArgs a)
{
    const int r = a.row_list ? a.row_list[bid_x()] : bid_x(), h = bid_y();
    const long long p0 = ((long long)r * a.H + h) * a.nsplit;
    const int lane = lane_id();
    // (nsplit <= 64: a lane per split; the sums of the first values are requested before the weights are known)
    const float m = lane < a.nsplit ? a.part_ml[(p0 + lane) * 2] : TA_NEG_BIG;
    const float l = lane < a.nsplit ? a.part_ml[(p0 + lane) * 2 + 1] : 0.0f;
    float pv[16];
    #pragma unroll
    for (int i = 0; i < 16; i++) pv[i] = a.part_o[(p0 + min(i, a.nsplit - 1)) * a.vdim + min(lane, a.vdim - 1)];
    const float mx = wave_allreduce_max(m);
    const float c = m > 0.5f * TA_NEG_BIG ? expf(m - mx) : 0.0f;
    const float lsum = wave_allreduce_add(l * c);
    const float inv = lsum > 0.0f ? 1.0f / lsum : 0.0f;
    for (int e0 = 0; e0 < a.vdim; e0 += 64)
    {
        const int e = e0 + lane, ec = min(e, a.vdim - 1);
        float o = 0.0f;
        for (int s0 = 0; s0 < a.nsplit; s0 += 16)
        {
            if (e0 + s0 > 0)
            {
                #pragma unroll
                for (int i = 0; i < 16; i++) pv[i] = a.part_o[(p0 + min(s0 + i, a.nsplit - 1)) * a.vdim + ec];
            }
            #pragma unroll
            for (int i = 0; i < 16; i++)
            {
                const float ci = shfl_idx_f32(c, min(s0 + i, 63));
                if (s0 + i < a.nsplit && ci > 0.0f) o = fmaf(pv[i], ci, o);
            }
        }
        if (e < a.vdim) ta_st<T>((T*)a.out + ((long long)r * a.H + h) * a.vdim + e, o * inv);
    }
}

// c tanh(s / c) by the hardware exponential and reciprocal (bfloat16 forms): 1 - 2 / (e^(2 s / c) + 1), absolute error a few 1e-7 c
DEV float tm_soft_cap(float s, float cap, float two_over_cap)
{
    return cap > 0.0f ? fmaf(-2.0f * cap, fast_rcp_approx(fast_exp(s * two_over_cap) + 1.0f), cap) : s;
}

DEV u32 tm_pack2(float lo, float hi) { return (u32)f32_to_bf16(lo) | ((u32)f32_to_bf16(hi) << 16); }

extern "C" int exl2_talk_attn_tiles_supported(int heads, int dim, int vdim);

// ---- bfloat16 on the matrix cores: decoded tokens -----------------------------------------------------------------------------------
// Workgroup = one row x all heads x one share of the keys, 32 keys at a time (one workgroup draws only so much from memory at once: few
// keys each, many workgroups), eight waves, up to 16 GPW heads over up to 4 GPW key / value heads.  Wave w scores keys 16 (w % 2) .. + 15
// for GPW key / value heads (A = key rows from the cache, B = the query heads that share them), the scores go to LDS as [head][key];
// then a half of a wave takes GPW heads with a key per lane: it mixes (T in LDS, transposed, read as broadcasts), joins the running
// softmax with lane exchanges and leaves the probabilities in LDS; last wave w adds V^T P^T of key / value head w (values through a
// wave-private LDS tile and transposing reads).  Keys and values of a step are all requested before its first product.

#define TD_NW 8
#define TD_BK 32
#define TD_STR 36                            // floats between two heads' scores
#define TD_TS 36                             // floats between two rows of T

// H <= 16 GPW heads, G <= 4 GPW key / value heads
template <int VDIM> HD size_t td_smem(int H)
{
    return sizeof(float) * ((size_t)2 * H * TD_STR + (size_t)H * TD_TS + ((3 * (size_t)H + 3) & ~(size_t)3)) + sizeof(u16) * (size_t)TD_NW * TD_BK * (VDIM + 16);
}

DEV float td_half_max(float v) { v = row16_allreduce_max(v); return fmaxf(v, shfl_xor_f32(v, 16)); }
DEV float td_half_sum(float v) { v = row16_allreduce_add(v); return v + shfl_xor_f32(v, 16); }

template <int DIM, int VDIM, int GPW>
KERNEL void __launch_bounds__(64 * TD_NW, 1) talk_attn_decode_kernel(const TalkArgs a)
{
    DYN_SMEM(smem);
    SHARED long long s_row[TD_BK];
    constexpr int KK = DIM / 32, DB = VDIM / 16, VSTR = VDIM + 16, VPR = VDIM / 8, VP = TD_BK * VPR / 64;
    constexpr int HQ = GPW;                                      // heads per half of a wave
    const int H = a.H, G = a.G, hpg = H / G;
    float* s_a = (float*)smem;                                   // [H][TD_STR] capped scores
    float* s_p = s_a + H * TD_STR;                               // [H][TD_STR] probabilities
    float* s_t = s_p + H * TD_STR;                               // [H (head in)][TD_TS]: T transposed, head out along the row
    float* s_c = s_t + H * TD_TS;                                // [H] correction of the step, [H] final maximum, [H] final sum
    u16* s_v = (u16*)(s_c + ((3 * H + 3) & ~3));                 // [TD_NW][TD_BK][VSTR], 16-byte aligned
    const int t = tid(), lane = lane_id();
    const int wv = uniform(wave_id());                           // (scalar branches around the matrix products: they ignore the lane mask)
    const int qi = lane & 15, g = lane >> 4;
    const int r = a.row_list ? a.row_list[bid_x()] : bid_x();
    const int split = bid_y();
    const int pos = a.row_pos[r];
    const int* bt = a.block_table + (long long)a.row_seq[r] * a.bt_stride;
    const int j_lo = max(0, pos - a.window + 1);
    const int total = pos - j_lo + 1;
    const int all_steps = (total + TD_BK - 1) / TD_BK;
    const int per_split = (all_steps + a.nsplit - 1) / a.nsplit;
    const int step0 = split * per_split, step1 = min(all_steps, step0 + per_split);
    const u16* kc = (const u16*)a.k_cache; const u16* vc = (const u16*)a.v_cache;
    u16* my_v = s_v + wv * TD_BK * VSTR;
    // T is requested first and put down behind the look-ups of the first step's rows (which take longer)
    constexpr int TL = (16 * GPW * 16 * GPW + 64 * TD_NW - 1) / (64 * TD_NW);
    float tv0[TL];
    #pragma unroll
    for (int i = 0; i < TL; i++) tv0[i] = a.talk[min(t + i * 64 * TD_NW, H * H - 1)];
    // the heads of this half wave in the mixing stage: hm .. + HQ - 1, key = lane % 32
    const int hm = (2 * wv + lane / 32) * HQ, key = lane % 32;
    float m_run[HQ], l_run[HQ];
    const bool with_sink = a.sink && split == 0;                 // the sink counts once
    #pragma unroll
    for (int i = 0; i < HQ; i++)
    {
        m_run[i] = with_sink ? a.sink[min(hm + i, H - 1)] : TA_NEG_BIG;
        l_run[i] = with_sink ? 1.0f : 0.0f;
    }
    f32x4 ot[DB];
    #pragma unroll
    for (int d = 0; d < DB; d++) ot[d] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    const float cap2 = a.softcap > 0.0f ? 2.0f / a.softcap : 0.0f;

    for (int step = step0; step < step1; step++)
    {
        const int k0 = step * TD_BK, nc = min(TD_BK, total - k0);
        const long long krow = ta_cache_row(a, bt, j_lo + k0 + min(16 * (wv % 2) + qi, nc - 1));
        if (t < TD_BK) s_row[t] = ta_cache_row(a, bt, j_lo + k0 + min(t, nc - 1));
        if (step == step0)
        {
            #pragma unroll
            for (int i = 0; i < TL; i++)
            {
                const int at = t + i * 64 * TD_NW;
                if (at < H * H) s_t[(at % H) * TD_TS + at / H] = tv0[i];
            }
        }
        u32x4 kf[GPW][KK], qf[GPW][KK], vreg[VP];
        const int g0 = (wv / 2) * GPW;
        #pragma unroll
        for (int k = 0; k < GPW; k++)
        {
            const int kv = min(g0 + k, G - 1);
            const u16* kp = kc + (krow * G + kv) * DIM + 8 * g;
            const u16* qp = (const u16*)a.q + ((long long)r * H + kv * hpg + min(qi, hpg - 1)) * DIM + 8 * g;
            #pragma unroll
            for (int kk = 0; kk < KK; kk++) { kf[k][kk] = *(const u32x4*)(kp + 32 * kk); qf[k][kk] = *(const u32x4*)(qp + 32 * kk); }
        }
        block_sync();                                            // (also: everybody is done with the previous step)
        #pragma unroll
        for (int i = 0; i < VP; i++)
            vreg[i] = *(const u32x4*)(vc + (s_row[(lane + 64 * i) / VPR] * G + min(wv, G - 1)) * VDIM + ((lane + 64 * i) % VPR) * 8);
        // ---- scores
        #pragma unroll
        for (int k = 0; k < GPW; k++)
        {
            if (g0 + k >= G) break;
            f32x4 st = {0.0f, 0.0f, 0.0f, 0.0f};
            #pragma unroll
            for (int kk = 0; kk < KK; kk++) st = mfma_16x16x32_bf16(kf[k][kk], qf[k][kk], st);
            #pragma unroll
            for (int e = 0; e < 4; e++) st[e] = tm_soft_cap(st[e], a.softcap, cap2);
            if (qi < hpg) *(f32x4*)(s_a + ((g0 + k) * hpg + qi) * TD_STR + 16 * (wv % 2) + 4 * g) = st;
        }
        block_sync_lds();
        // ---- the exchange between the heads and the softmax: lane = key
        if (2 * wv * HQ < H)
        {
            float mx[HQ];
            #pragma unroll
            for (int i = 0; i < HQ; i++) mx[i] = 0.0f;
            #pragma unroll 8
            for (int c = 0; c < H; c++)
            {
                const float sv = s_a[c * TD_STR + key];
                #pragma unroll
                for (int i = 0; i < HQ; i++) mx[i] = fmaf(s_t[c * TD_TS + hm + i], sv, mx[i]);       // (columns past H are never used)
            }
            #pragma unroll
            for (int i = 0; i < HQ; i++)
            {
                const float s = key < nc ? mx[i] : TA_NEG_BIG;
                const float m_new = fmaxf(m_run[i], td_half_max(s));
                const float p = key < nc ? fast_exp(s - m_new) : 0.0f;
                const float c = fast_exp(m_run[i] - m_new);
                l_run[i] = l_run[i] * c + td_half_sum(p);
                m_run[i] = m_new;
                if (hm + i < H)
                {
                    s_p[(hm + i) * TD_STR + key] = p;
                    if (key == 0) s_c[hm + i] = c;
                }
            }
        }
        block_sync_lds();
        // ---- values: this wave's key / value head
        if (wv < G)
        {
            const int h = wv * hpg + min(qi, hpg - 1);
            const float alpha = s_c[h];
            ta_wave_lds();
            #pragma unroll
            for (int i = 0; i < VP; i++) *(u32x4*)(my_v + ((lane + 64 * i) / VPR) * VSTR + ((lane + 64 * i) % VPR) * 8) = vreg[i];
            ta_wave_lds();
            const u16* vbase = my_v + (4 * g + (qi >> 2)) * VSTR + 4 * (qi & 3);
            const f32x4 pa = *(const f32x4*)(s_p + h * TD_STR + 4 * g), pc = *(const f32x4*)(s_p + h * TD_STR + 16 + 4 * g);
            const u32x4 pb = {tm_pack2(pa[0], pa[1]), tm_pack2(pa[2], pa[3]), tm_pack2(pc[0], pc[1]), tm_pack2(pc[2], pc[3])};
            #pragma unroll
            for (int d = 0; d < DB; d++)
            {
                #pragma unroll
                for (int e = 0; e < 4; e++) ot[d][e] *= alpha;
                const f16x4 lo = lds_read_tr16_b64((const f16*)(vbase + 16 * d));
                const f16x4 hi = lds_read_tr16_b64((const f16*)(vbase + 16 * VSTR + 16 * d));
                const u32x2 l2 = __builtin_bit_cast(u32x2, lo), h2 = __builtin_bit_cast(u32x2, hi);
                ot[d] = mfma_16x16x32_bf16((u32x4){l2[0], l2[1], h2[0], h2[1]}, pb, ot[d]);
            }
        }
    }
    #pragma unroll
    for (int i = 0; i < HQ; i++)
    {
        const int h = hm + i;
        if (h < H && key == 0)
        {
            s_c[H + h] = m_run[i];
            s_c[2 * H + h] = l_run[i];
            if (a.nsplit > 1)
            {
                const long long pi = ((long long)r * H + h) * a.nsplit + split;
                a.part_ml[pi * 2] = m_run[i]; a.part_ml[pi * 2 + 1] = l_run[i];
            }
        }
    }
    block_sync();
    if (wv >= G || qi >= hpg) return;
    const int h = wv * hpg + qi;
    if (a.nsplit > 1)
    {
        float* po = a.part_o + (((long long)r * H + h) * a.nsplit + split) * VDIM + 4 * g;
        #pragma unroll
        for (int d = 0; d < DB; d++) *(f32x4*)(po + 16 * d) = ot[d];
    }
    else
    {
        const float l = s_c[2 * H + h], inv = l > 0.0f ? 1.0f / l : 0.0f;
        u16* op = (u16*)a.out + ((long long)r * H + h) * VDIM + 4 * g;
        #pragma unroll
        for (int d = 0; d < DB; d++)
            *(u32x2*)(op + 16 * d) = (u32x2){tm_pack2(ot[d][0] * inv, ot[d][1] * inv), tm_pack2(ot[d][2] * inv, ot[d][3] * inv)};
    }
}

template <int DIM, int VDIM, int GPW>
static void td_launch_one(const TalkArgs& a, int rows, hipStream_t s)
{
    static bool attr_done[EXL2_MAX_DEVICES];
    if (exl2_first_on_device(attr_done))
        (void)hipFuncSetAttribute((const void*)talk_attn_decode_kernel<DIM, VDIM, GPW>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024);
    LAUNCH((talk_attn_decode_kernel<DIM, VDIM, GPW>), dim3(rows, a.nsplit), dim3(64 * TD_NW), td_smem<VDIM>(a.H), s, a);
}

template <int DIM, int VDIM>
static void td_launch(const TalkArgs& a, int rows, hipStream_t s)
{
    if (a.H <= 16 && a.G <= 4) td_launch_one<DIM, VDIM, 1>(a, rows, s);
    else td_launch_one<DIM, VDIM, 2>(a, rows, s);
}

// ---- bfloat16 on the matrix cores: portions of prompts -----------------------------------------------------------------------------
// Workgroup = one tile of <= 16 consecutive positions of one sequence x 16 output heads x one share of the key steps, eight waves.  Keys
// go by 32 at a time in three stages (heads in quads of four consecutive ones; HB = 1: up to 16 heads, 2: up to 32, two workgroups):
//   1. scores of ALL heads, S^T = K Q^T: a wave takes a quad and all 32 keys (HB = 2) or half of them (A = key rows straight from the
//      cache: a lane's 8 values are one 16-byte load that feeds every head of the quad with the same key / value head), capped, to LDS
//      as fp32 [head][query][key];
//   2. the exchange: a lane takes one (query, key), s_h = sum_g T[h, g] a_g -- on the fp32 matrix cores in their 16-block form, where
//      every lane's own scalar goes through a 4 x 1 product per (four heads out, one head in) without any lane movement -- and puts the
//      mixed scores of the 16 output heads back in place;
//   3. the output heads, two waves per quad: online softmax (columns = queries), probabilities to bfloat16 in registers (the accumulator layout of S^T is the
//      operand layout of O^T += V^T P^T with the keys of a product taken in the order {4 g .. + 3 of block 0, of block 1}); the two waves
//      take half of the value columns each, through a wave-private LDS tile and transposing reads.
// The step's value rows are requested before stage 2, the next step's key rows before stage 3; the rows' places in the cache are looked
// up by one wave a step ahead.

#define TM_Q 16
#define TM_NW 8
#define TM_BK 32
#define TM_MAX_SPLIT 8

template <int DIM, int VDIM, int HB>
struct TalkTile
{
    static constexpr int HMAX = 16 * HB, SS = TM_BK + 4, TS = HMAX + 4, VW = VDIM / 2, VSTR = VW + 16;
    static constexpr size_t smem = sizeof(float) * ((size_t)HMAX * TM_Q * SS + (size_t)16 * TS) + sizeof(u16) * (size_t)TM_NW * TM_BK * VSTR;
};

template <int DIM, int VDIM, int HB>
KERNEL void __launch_bounds__(64 * TM_NW, 1) talk_attn_tile_kernel(const TalkArgs a)
{
    DYN_SMEM(smem);
    SHARED int s_row[2][TM_BK];
    typedef TalkTile<DIM, VDIM, HB> TT;
    constexpr int SS = TT::SS, TS = TT::TS, VSTR = TT::VSTR, VW = TT::VW, KB = HB, KK = DIM / 32, DB = VW / 16;
    constexpr int VPR = VW / 8, VP = TM_BK * VPR / 64;           // 16-byte pieces of a wave's part of a value row; pieces per lane
    constexpr int NT = 4;                                        // groups of four heads out
    float* s_s = (float*)smem;                                   // [HMAX][TM_Q][SS]
    float* s_t = s_s + TT::HMAX * TM_Q * SS;                     // [16][TS]: T's rows of the output heads, zero past H
    u16* s_v = (u16*)(s_t + 16 * TS);                            // [TM_NW][TM_BK][VSTR]

    const int t = tid(), lane = lane_id();
    const int wv = uniform(wave_id());                           // (scalar branches around the matrix products: they ignore the lane mask)
    const int og = bid_z() * 16;                                 // first output head of the workgroup
    const int quad1 = HB == 1 ? wv / 2 : wv, kpart = HB == 1 ? wv % 2 : 0;       // stage 1: quad of heads, first 16-key block
    const int part = wv % 2;                                     // stage 3: half of the value columns
    const int qi = lane & 15, g = lane >> 4;
    const int H = a.H, G = a.G, hpg = H / G;
    const int tile_i = gdim_x() - 1 - bid_x(), split = bid_y();  // the longest key lists first
    const int r0 = a.tile_row0[tile_i], n_rows = a.tile_rows[tile_i];
    const int p0 = a.row_pos[r0], p_last = p0 + n_rows - 1;
    const int* bt = a.block_table + (long long)a.row_seq[r0] * a.bt_stride;
    const int j_lo = max(0, p0 - a.window + 1);
    const int total = p_last - j_lo + 1;
    const int all_steps = (total + TM_BK - 1) / TM_BK;
    const int per_split = (all_steps + a.nsplit - 1) / a.nsplit;
    const int step0 = split * per_split, step1 = min(all_steps, step0 + per_split);
    const u16* kc = (const u16*)a.k_cache; const u16* vc = (const u16*)a.v_cache;
    u16* my_v = s_v + wv * TM_BK * VSTR;
    const float cap2 = a.softcap > 0.0f ? 2.0f / a.softcap : 0.0f;

    const int nq = max(0, min(4, H - 4 * quad1)), q0 = min(4 * quad1, H - 1);                        // stage 1: heads of this wave
    const int nh = max(0, min(4, H - og - 4 * (wv / 2))), h0 = min(og + 4 * (wv / 2), H - 1);        // stage 3
    int kvq[4], kvh[4];
    #pragma unroll
    for (int n = 0; n < 4; n++) { kvq[n] = uniform(min(q0 + n, H - 1) / hpg); kvh[n] = uniform(min(h0 + n, H - 1) / hpg); }

    const int qrow = r0 + min(qi, n_rows - 1), qpos = p0 + min(qi, n_rows - 1), q_lo = qpos - a.window + 1;
    u32x4 qb[4][KK];
    f32x4 ot[4][DB];
    float m_run[4], l_run[4];
    const bool with_sink = a.sink && split == 0;                 // the sink counts once
    #pragma unroll
    for (int n = 0; n < 4; n++)
    {
        const int h = min(h0 + n, H - 1);
        const u16* qp = (const u16*)a.q + ((long long)qrow * H + min(q0 + n, H - 1)) * DIM + 8 * g;
        #pragma unroll
        for (int kk = 0; kk < KK; kk++) qb[n][kk] = *(const u32x4*)(qp + 32 * kk);
        #pragma unroll
        for (int d = 0; d < DB; d++) ot[n][d] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
        m_run[n] = with_sink ? a.sink[h] : TA_NEG_BIG;
        l_run[n] = with_sink && g == 0 ? 1.0f : 0.0f;            // (a lane's own share: the four lanes of a query add theirs up at the end)
    }
    u32x4 kf[KB][KK], vreg[VP];
    auto load_k = [&](int step, int kv) {
        #pragma unroll
        for (int b = 0; b < KB; b++)
        {
            const u16* kp = kc + ((long long)s_row[step & 1][16 * (kpart + b) + qi] * G + kv) * DIM + 8 * g;
            #pragma unroll
            for (int kk = 0; kk < KK; kk++) kf[b][kk] = *(const u32x4*)(kp + 32 * kk);
        }
    };
    auto load_v = [&](int step, int kv) {
        #pragma unroll
        for (int i = 0; i < VP; i++)
            vreg[i] = *(const u32x4*)(vc + ((long long)s_row[step & 1][(lane + 64 * i) / VPR] * G + kv) * VDIM + part * VW + ((lane + 64 * i) % VPR) * 8);
    };
    if (step0 < step1)
    {
        for (int i = t; i < 16 * TT::HMAX; i += 64 * TM_NW)
        {
            const int h = i / TT::HMAX, c = i % TT::HMAX;
            s_t[h * TS + c] = og + h < H && c < H ? a.talk[(og + h) * H + c] : 0.0f;
        }
        if (t < TM_BK) s_row[step0 & 1][t] = (int)ta_cache_row(a, bt, j_lo + min(step0 * TM_BK + t, total - 1));
        block_sync();
        if (nq > 0) load_k(step0, kvq[0]);
    }

    for (int step = step0; step < step1; step++)
    {
        const int k0 = step * TM_BK;
        int next_row = 0;
        if (t < TM_BK) next_row = (int)ta_cache_row(a, bt, j_lo + min(k0 + TM_BK + t, total - 1));
        // ---- 1: scores of the quad's heads
        #pragma unroll
        for (int n = 0; n < 4; n++)
        {
            if (n >= nq) break;
            if (n > 0 && kvq[n] != kvq[n - 1]) load_k(step, kvq[n]);
            float* sr = s_s + ((q0 + n) * TM_Q + qi) * SS + 16 * kpart + 4 * g;
            #pragma unroll
            for (int b = 0; b < KB; b++)
            {
                f32x4 st = {0.0f, 0.0f, 0.0f, 0.0f};
                #pragma unroll
                for (int kk = 0; kk < KK; kk++) st = mfma_16x16x32_bf16(kf[b][kk], qb[n][kk], st);
                #pragma unroll
                for (int r = 0; r < 4; r++) st[r] = tm_soft_cap(st[r], a.softcap, cap2);
                *(f32x4*)(sr + 16 * b) = st;
            }
        }
        block_sync_lds();
        if (nh > 0) load_v(step, kvh[0]);
        // (the other half of the table held the step before this one: every wave is past it)
        if (t < TM_BK) s_row[(step + 1) & 1][t] = next_row;
        // ---- 2: the exchange between the heads, in place
        {
            float* sp = s_s + (t / TM_BK) * SS + t % TM_BK;
            f32x4 mx[NT];
            #pragma unroll
            for (int i = 0; i < NT; i++) mx[i] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
            for (int c = 0; c < H; c += 4)
            {
                f32x4 tv[NT];
                float sv[4];
                #pragma unroll
                for (int k = 0; k < 4; k++) sv[k] = sp[min(c + k, H - 1) * TM_Q * SS];          // (past the last head T is zero)
                #pragma unroll
                for (int i = 0; i < NT; i++) tv[i] = *(const f32x4*)(s_t + (4 * i + (lane & 3)) * TS + c);
                #pragma unroll
                for (int k = 0; k < 4; k++)
                    #pragma unroll
                    for (int i = 0; i < NT; i++) mx[i] = mfma_4x4x1_f32(tv[i][k], sv[k], mx[i]);
            }
            #pragma unroll
            for (int i = 0; i < NT; i++)
                #pragma unroll
                for (int r = 0; r < 4; r++)
                    if (4 * i + r < H - og) sp[(4 * i + r) * TM_Q * SS] = mx[i][r];
        }
        block_sync_lds();
        // ---- 3: softmax and values of the quad's heads
        if (nq > 0 && step + 1 < step1) load_k(step + 1, kvq[0]);
        if (nh > 0)
        {
            u32x4 pb[4];
            float alpha[4];
            bool moved = false;
            #pragma unroll
            for (int n = 0; n < 4; n++)
            {
                alpha[n] = 1.0f;
                if (n >= nh) break;
                const float* sr = s_s + ((h0 - og + n) * TM_Q + qi) * SS + 4 * g;
                float sc[8];
                float m_loc = TA_NEG_BIG;
                #pragma unroll
                for (int b = 0; b < 2; b++)
                {
                    const f32x4 v = *(const f32x4*)(sr + 16 * b);
                    #pragma unroll
                    for (int r = 0; r < 4; r++)
                    {
                        const int j = j_lo + k0 + 16 * b + 4 * g + r;
                        sc[4 * b + r] = j <= qpos && j >= q_lo ? v[r] : TA_NEG_BIG;
                        m_loc = fmaxf(m_loc, sc[4 * b + r]);
                    }
                }
                m_loc = fmaxf(m_loc, shfl_xor_f32(m_loc, 16));
                m_loc = fmaxf(m_loc, shfl_xor_f32(m_loc, 32));
                const float m_new = fmaxf(m_run[n], m_loc);
                alpha[n] = fast_exp(m_run[n] - m_new);
                moved = moved || alpha[n] != 1.0f;
                float p_sum = 0.0f;
                #pragma unroll
                for (int e2 = 0; e2 < 4; e2++)
                {
                    const float pa = sc[2 * e2] > 0.5f * TA_NEG_BIG ? fast_exp(sc[2 * e2] - m_new) : 0.0f;
                    const float pc = sc[2 * e2 + 1] > 0.5f * TA_NEG_BIG ? fast_exp(sc[2 * e2 + 1] - m_new) : 0.0f;
                    p_sum += pa + pc;
                    pb[n][e2] = tm_pack2(pa, pc);
                }
                l_run[n] = l_run[n] * alpha[n] + p_sum;
                m_run[n] = m_new;
            }
            if (wave_ballot(moved) != 0ull)                      // the running maxima rarely move once a few steps have gone by
            {
                #pragma unroll
                for (int n = 0; n < 4; n++)
                    #pragma unroll
                    for (int d = 0; d < DB; d++)
                        #pragma unroll
                        for (int e = 0; e < 4; e++) ot[n][d][e] *= alpha[n];
            }
            // runs of heads that read the same key / value head: its values once through LDS, every fragment feeds all of the run
            #pragma unroll
            for (int n0 = 0; n0 < 4; n0++)
            {
                if (n0 >= nh) break;
                if (n0 > 0 && kvh[n0] == kvh[n0 - 1]) continue;
                if (n0 > 0) load_v(step, kvh[n0]);
                ta_wave_lds();
                #pragma unroll
                for (int i = 0; i < VP; i++) *(u32x4*)(my_v + ((lane + 64 * i) / VPR) * VSTR + ((lane + 64 * i) % VPR) * 8) = vreg[i];
                ta_wave_lds();
                const u16* vbase = my_v + (4 * g + (qi >> 2)) * VSTR + 4 * (qi & 3);
                #pragma unroll
                for (int d = 0; d < DB; d++)
                {
                    const f16x4 lo = lds_read_tr16_b64((const f16*)(vbase + 16 * d));
                    const f16x4 hi = lds_read_tr16_b64((const f16*)(vbase + 16 * VSTR + 16 * d));
                    const u32x2 l2 = __builtin_bit_cast(u32x2, lo), h2 = __builtin_bit_cast(u32x2, hi);
                    #pragma unroll
                    for (int n = n0; n < 4; n++)
                        if (n < nh && kvh[n] == kvh[n0]) ot[n][d] = mfma_16x16x32_bf16((u32x4){l2[0], l2[1], h2[0], h2[1]}, pb[n], ot[n][d]);
                }
            }
        }
        block_sync_lds();                                        // stage 1 of the next step overwrites the scores
    }

    #pragma unroll
    for (int n = 0; n < 4; n++)
    {
        l_run[n] += shfl_xor_f32(l_run[n], 16);
        l_run[n] += shfl_xor_f32(l_run[n], 32);
    }
    if (qi >= n_rows) return;
    #pragma unroll
    for (int n = 0; n < 4; n++)
    {
        if (n >= nh) break;
        if (a.nsplit > 1)
        {
            const long long pi = ((long long)qrow * H + h0 + n) * a.nsplit + split;
            float* po = a.part_o + pi * VDIM + part * VW + 4 * g;
            #pragma unroll
            for (int d = 0; d < DB; d++) *(f32x4*)(po + 16 * d) = ot[n][d];
            if (part == 0 && g == 0) { a.part_ml[pi * 2] = m_run[n]; a.part_ml[pi * 2 + 1] = l_run[n]; }
            continue;
        }
        const float inv = l_run[n] > 0.0f ? 1.0f / l_run[n] : 0.0f;
        u16* op = (u16*)a.out + ((long long)qrow * H + h0 + n) * VDIM + part * VW + 4 * g;
        #pragma unroll
        for (int d = 0; d < DB; d++)
            *(u32x2*)(op + 16 * d) = (u32x2){tm_pack2(ot[n][d][0] * inv, ot[n][d][1] * inv), tm_pack2(ot[n][d][2] * inv, ot[n][d][3] * inv)};
    }
}

// grid (tiles, heads): joins the key splits of a tile's rows; thread = (row, four values)
KERNEL void __launch_bounds__(256) talk_attn_tile_merge_kernel(const TalkArgs a)
{
    const int r0 = a.tile_row0[bid_x()], n_rows = a.tile_rows[bid_x()], h = bid_y(), per = a.vdim / 4;
    for (int i = tid(); i < n_rows * per; i += 256)
    {
        const int row = r0 + i / per, e = (i % per) * 4;
        const long long p0 = ((long long)row * a.H + h) * a.nsplit;
        float m[TM_MAX_SPLIT], l[TM_MAX_SPLIT];
        f32x4 o[TM_MAX_SPLIT];
        float mx = TA_NEG_BIG;
        #pragma unroll
        for (int s = 0; s < TM_MAX_SPLIT; s++)
        {
            const long long p = p0 + min(s, a.nsplit - 1);
            m[s] = a.part_ml[p * 2];
            l[s] = a.part_ml[p * 2 + 1];
            o[s] = *(const f32x4*)(a.part_o + p * a.vdim + e);
        }
        #pragma unroll
        for (int s = 0; s < TM_MAX_SPLIT; s++) mx = fmaxf(mx, m[s]);
        float lsum = 0.0f;
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        #pragma unroll
        for (int s = 0; s < TM_MAX_SPLIT; s++)
        {
            if (s >= a.nsplit || m[s] <= 0.5f * TA_NEG_BIG) continue;
            const float c = fast_exp(m[s] - mx);
            lsum = fmaf(l[s], c, lsum);
            #pragma unroll
            for (int k = 0; k < 4; k++) acc[k] = fmaf(o[s][k], c, acc[k]);
        }
        const float inv = lsum > 0.0f ? 1.0f / lsum : 0.0f;
        *(u32x2*)((u16*)a.out + ((long long)row * a.H + h) * a.vdim + e) = (u32x2){tm_pack2(acc[0] * inv, acc[1] * inv), tm_pack2(acc[2] * inv, acc[3] * inv)};
    }
}

template <int DIM, int VDIM, int HB>
static void tm_launch_one(const TalkArgs& a, int tiles, hipStream_t s)
{
    static bool attr_done[EXL2_MAX_DEVICES];
    static_assert(TalkTile<DIM, VDIM, HB>::smem <= 159 * 1024, "the tile fits the LDS");
    if (exl2_first_on_device(attr_done))
        (void)hipFuncSetAttribute((const void*)talk_attn_tile_kernel<DIM, VDIM, HB>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024);
    LAUNCH((talk_attn_tile_kernel<DIM, VDIM, HB>), dim3(tiles, a.nsplit, HB), dim3(64 * TM_NW), (TalkTile<DIM, VDIM, HB>::smem), s, a);
    if (a.nsplit > 1) LAUNCH(talk_attn_tile_merge_kernel, dim3(tiles, a.H), dim3(256), 0, s, a);
}

template <int DIM, int VDIM>
static void tm_launch(const TalkArgs& a, int tiles, hipStream_t s)
{
    if (a.H <= 16) tm_launch_one<DIM, VDIM, 1>(a, tiles, s);
    else tm_launch_one<DIM, VDIM, 2>(a, tiles, s);
}

// ---- C ABI ----------------------------------------------------------------------------------------------------------------------

static int ta_log2_exact(int x) { int sh = 0; while ((1 << sh) < x) sh++; return x > 0 && (1 << sh) == x ? sh : -1; }

/* 1 if exl2_talk_attn_tiles takes these sizes (bfloat16) */
extern "C" int exl2_talk_attn_tiles_supported(int heads, int dim, int vdim)
{
    return heads <= 32 && ((dim == 32 && vdim == 32) || ((dim == 64 || dim == 128) && (vdim == 64 || vdim == 128)));
}

static int ta_fill(TalkArgs& a, const void* q, const void* k_cache, const void* v_cache, const float* talk, const float* sink,
                   const int* row_seq, const int* row_pos, const int* block_table, int bt_stride, int page, void* out, int heads,
                   int kv_heads, int dim, int vdim, int window, float softcap)
{
    EXL2_REQUIRE(q && k_cache && v_cache && talk && row_seq && row_pos && block_table && out, "talk_attn: null operand");
    EXL2_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, "talk_attn: bad head shape");
    EXL2_REQUIRE(page > 0 && window > 0 && softcap >= 0.0f, "talk_attn: bad window / paging / soft cap");
    a.q = q; a.k_cache = k_cache; a.v_cache = v_cache; a.talk = talk; a.sink = sink; a.row_seq = row_seq; a.row_pos = row_pos;
    a.block_table = block_table; a.bt_stride = bt_stride; a.page = page; a.page_shift = ta_log2_exact(page); a.out = out; a.H = heads;
    a.G = kv_heads; a.dim = dim; a.vdim = vdim; a.window = window; a.softcap = softcap; a.row_list = nullptr; a.tile_row0 = nullptr;
    a.tile_rows = nullptr; a.part_o = nullptr; a.part_ml = nullptr; a.nsplit = 1;
    return EXL2_OK;
}

extern "C" int exl2_talk_attn(const void* q, const void* k_cache, const void* v_cache, const float* talk, const float* sink,
                              const int* row_seq, const int* row_pos, const int* block_table, int bt_stride, int page, void* out,
                              const int* row_list, int rows, float* part_o, float* part_ml, int nsplit, int dtype, int heads, int kv_heads,
                              int dim, int vdim, int window, float softcap, void* stream)
{
    TalkArgs a;
    const int rc = ta_fill(a, q, k_cache, v_cache, talk, sink, row_seq, row_pos, block_table, bt_stride, page, out, heads, kv_heads, dim,
                           vdim, window, softcap);
    if (rc != EXL2_OK) return rc;
    EXL2_REQUIRE(dtype == 0 || dtype == 1, "talk_attn: dtype must be 0 (bfloat16) or 1 (float32)");
    EXL2_REQUIRE(nsplit >= 1 && nsplit <= TA_MAX_SPLIT && (nsplit == 1 || (part_o && part_ml)), "talk_attn: key splits (1 .. %d) need scratch", TA_MAX_SPLIT);
    const size_t smem = ta_row_smem(heads, dim, vdim);
    if (smem + 1024 > 160 * 1024)
        EXL2_FAIL(EXL2_E_UNSUPPORTED, "talk_attn: %d heads of %d / %d values do not fit the LDS", heads, dim, vdim);
    if (rows <= 0) return EXL2_OK;
    a.row_list = row_list; a.part_o = part_o; a.part_ml = part_ml; a.nsplit = nsplit;
    const int vn = dtype == 0 ? 8 : 4;
    const bool vec = dim % vn == 0 && vdim % 2 == 0 && ((uintptr_t)k_cache % 16) == 0 && ((uintptr_t)v_cache % 8) == 0;
    hipStream_t s = (hipStream_t)stream;
    if (dtype == 0 && vec && row_list && exl2_talk_attn_tiles_supported(heads, dim, vdim) && kv_heads <= 8 && heads / kv_heads <= 16
        && ((uintptr_t)q % 16) == 0 && ((uintptr_t)v_cache % 16) == 0 && ((uintptr_t)part_o % 16) == 0 && ((uintptr_t)out % 8) == 0)
    {
        // listed rows (decoded tokens) at the sizes of the matrix-core form
        if (dim == 32) td_launch<32, 32>(a, rows, s);
        else if (dim == 64 && vdim == 64) td_launch<64, 64>(a, rows, s);
        else if (dim == 64) td_launch<64, 128>(a, rows, s);
        else if (vdim == 64) td_launch<128, 64>(a, rows, s);
        else td_launch<128, 128>(a, rows, s);
        if (nsplit > 1) LAUNCH(talk_attn_merge_kernel<u16>, dim3(rows, heads), dim3(64), 0, stream, a);
        HIP_TRY(hipGetLastError());
        return EXL2_OK;
    }
    static bool attr_done[EXL2_MAX_DEVICES];
    if (exl2_first_on_device(attr_done))
    {
        (void)hipFuncSetAttribute((const void*)talk_attn_row_kernel<u16, true>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024);
        (void)hipFuncSetAttribute((const void*)talk_attn_row_kernel<u16, false>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024);
        (void)hipFuncSetAttribute((const void*)talk_attn_row_kernel<float, true>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024);
        (void)hipFuncSetAttribute((const void*)talk_attn_row_kernel<float, false>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 1024);
    }
    const dim3 grid(rows, nsplit);
    if (dtype == 0)
    {
        if (vec) LAUNCH((talk_attn_row_kernel<u16, true>), grid, dim3(256), smem, stream, a);
        else LAUNCH((talk_attn_row_kernel<u16, false>), grid, dim3(256), smem, stream, a);
        if (nsplit > 1) LAUNCH(talk_attn_merge_kernel<u16>, dim3(rows, heads), dim3(64), 0, stream, a);
    }
    else
    {
        if (vec) LAUNCH((talk_attn_row_kernel<float, true>), grid, dim3(256), smem, stream, a);
        else LAUNCH((talk_attn_row_kernel<float, false>), grid, dim3(256), smem, stream, a);
        if (nsplit > 1) LAUNCH(talk_attn_merge_kernel<float>, dim3(rows, heads), dim3(64), 0, stream, a);
    }
    HIP_TRY(hipGetLastError());
    return EXL2_OK;
}

extern "C" int exl2_talk_attn_tiles(const void* q, const void* k_cache, const void* v_cache, const float* talk, const float* sink,
                                    const int* row_seq, const int* row_pos, const int* block_table, int bt_stride, int page, void* out,
                                    const int* tile_row0, const int* tile_rows, int tiles, float* part_o, float* part_ml, int nsplit,
                                    int heads, int kv_heads, int dim, int vdim, int window, float softcap, void* stream)
{
    TalkArgs a;
    const int rc = ta_fill(a, q, k_cache, v_cache, talk, sink, row_seq, row_pos, block_table, bt_stride, page, out, heads, kv_heads, dim,
                           vdim, window, softcap);
    if (rc != EXL2_OK) return rc;
    EXL2_REQUIRE(tile_row0 && tile_rows, "talk_attn_tiles: tiles missing");
    if (!exl2_talk_attn_tiles_supported(heads, dim, vdim))
        EXL2_FAIL(EXL2_E_UNSUPPORTED, "talk_attn_tiles: %d heads of %d / %d values outside the matrix-core form", heads, dim, vdim);
    EXL2_REQUIRE(nsplit >= 1 && nsplit <= TM_MAX_SPLIT && (nsplit == 1 || (part_o && part_ml && ((uintptr_t)part_o % 16) == 0)),
                 "talk_attn_tiles: key splits (1 .. %d) need scratch", TM_MAX_SPLIT);
    if (tiles <= 0) return EXL2_OK;
    a.tile_row0 = tile_row0; a.tile_rows = tile_rows; a.part_o = part_o; a.part_ml = part_ml; a.nsplit = nsplit;
    hipStream_t s = (hipStream_t)stream;
    if (dim == 32) tm_launch<32, 32>(a, tiles, s);
    else if (dim == 64 && vdim == 64) tm_launch<64, 64>(a, tiles, s);
    else if (dim == 64) tm_launch<64, 128>(a, tiles, s);
    else if (vdim == 64) tm_launch<128, 64>(a, tiles, s);
    else tm_launch<128, 128>(a, tiles, s);
    HIP_TRY(hipGetLastError());
    return EXL2_OK;
}
