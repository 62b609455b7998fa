// mingru.hip -- a gated recurrence over one number per channel whose gates read only the current token (minimal GRU), for gfx950,
// + its C ABI.
//
// Per channel, with the projections z', u, g of the token (fp32, biases already added):
//     z = sigmoid(z'),   c = u + 1/2 where u >= 0, sigmoid(u) elsewhere,   S <- (1 - z) S + z c,   out = S silu(g)
// S is fp32, one per (slot, channel).  Channels never meet, so a step is a thread per channel; long spans are cut into chunks of
// tokens: a chunk maps the state as S -> a S + b, one launch makes every chunk's (a, b), a second one composes the maps in front of
// each chunk and walks its tokens again with the state they give.
//
// Rows of a step are a flat list; a span is the run of consecutive rows one sequence brings (span i = rows span_row0[i] ..
// + span_rows[i], slot and first position = row_seq / row_pos of its first row).  A span at position 0 starts from zeros whatever
// its slot holds.
#include "hw.h"
#include "errors.h"
#include <stdint.h>

template <typename T> DEV void mg_st(T* p, float v);
template <> DEV void mg_st<u16>(u16* p, float v) { *p = f32_to_bf16(v); }
template <> DEV void mg_st<float>(float* p, float v) { *p = v; }

DEV float mg_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
// one minus the gate from the gate's own argument (no cancellation where the gate is nearly 1)
DEV float mg_keep(float z) { return 1.0f / (1.0f + expf(z)); }
DEV float mg_candidate(float u) { return u >= 0.0f ? u + 0.5f : mg_sigmoid(u); }

#define MG_UNROLL 8                          // tokens whose inputs are requested together

struct MinGruArgs
{
    const float* z; const float* u; const float* g; int ld;      // [rows, ld] each (columns of one projection)
    void* out; int ldo;                      // [rows, ldo] operand dtype
    float* state;                            // [slots, width]
    const int* span_row0; const int* span_rows; const int* row_seq; const int* row_pos; int spans;
    const int* span_chunk0; int chunk;       // chunks in front of each span; tokens per chunk
    float* agg_a; float* agg_b;              // [chunks, width]
    float* s0;                               // [spans, width]: the state the span starts from
    int width;
};

// walks `n` tokens from row r; WRITE: leaves the outputs; returns S (and, in a, the product of the keep factors)
template <typename T, bool WRITE>
DEV float mg_walk(const MinGruArgs& m, int r, int n, int c, float S, float& a)
{
    for (int i0 = 0; i0 < n; i0 += MG_UNROLL)
    {
        float zv[MG_UNROLL], uv[MG_UNROLL], gv[MG_UNROLL];
        #pragma unroll
        for (int i = 0; i < MG_UNROLL; i++)
        {
            const long long at = (long long)(r + min(i0 + i, n - 1)) * m.ld + c;
            zv[i] = m.z[at];
            uv[i] = m.u[at];
            gv[i] = WRITE ? m.g[at] : 0.0f;
        }
        #pragma unroll
        for (int i = 0; i < MG_UNROLL; i++)
        {
            if (i0 + i >= n) break;
            const float keep = mg_keep(zv[i]);
            S = fmaf(keep, S, mg_sigmoid(zv[i]) * mg_candidate(uv[i]));
            a *= keep;
            if (WRITE) mg_st<T>((T*)m.out + (long long)(r + i0 + i) * m.ldo + c, S * gv[i] * mg_sigmoid(gv[i]));
        }
    }
    return S;
}

// grid (channel blocks, spans): decoded tokens and short portions
template <typename T>
KERNEL void __launch_bounds__(256) mingru_kernel(const MinGruArgs m)
{
    const int c = bid_x() * 256 + tid(), sp = bid_y();
    if (c >= m.width) return;
    const int r0 = m.span_row0[sp];
    float* st = m.state + (long long)m.row_seq[r0] * m.width + c;
    float a = 1.0f;
    *st = mg_walk<T, true>(m, r0, m.span_rows[sp], c, m.row_pos[r0] > 0 ? *st : 0.0f, a);
}

DEV int mg_span_of(const MinGruArgs& m, int chunk)
{
    int sp = 0;
    while (sp + 1 < m.spans && m.span_chunk0[sp + 1] <= chunk) sp++;
    return sp;
}

// grid (channel blocks, chunks): the chunk's map S -> a S + b
template <typename T>
KERNEL void __launch_bounds__(256) mingru_chunk_kernel(const MinGruArgs m)
{
    const int c = bid_x() * 256 + tid(), ch = bid_y();
    if (c >= m.width) return;
    const int sp = mg_span_of(m, ch), k = ch - m.span_chunk0[sp];
    const int r0 = m.span_row0[sp];
    const int n = min(m.chunk, m.span_rows[sp] - k * m.chunk);
    // the last launch overwrites the slot while others still need what the span starts from: it is put aside here
    if (k == 0) m.s0[(long long)sp * m.width + c] = m.row_pos[r0] > 0 ? m.state[(long long)m.row_seq[r0] * m.width + c] : 0.0f;
    float a = 1.0f;
    const float b = mg_walk<T, false>(m, r0 + k * m.chunk, n, c, 0.0f, a);
    m.agg_a[(long long)ch * m.width + c] = a;
    m.agg_b[(long long)ch * m.width + c] = b;
}

// grid (channel blocks, chunks): the state in front of the chunk, then its tokens; the span's last chunk leaves the slot's state
template <typename T>
KERNEL void __launch_bounds__(256) mingru_out_kernel(const MinGruArgs m)
{
    const int c = bid_x() * 256 + tid(), ch = bid_y();
    if (c >= m.width) return;
    const int sp = mg_span_of(m, ch), first = m.span_chunk0[sp], k = ch - first;
    const int r0 = m.span_row0[sp];
    const int n_tok = m.span_rows[sp], n = min(m.chunk, n_tok - k * m.chunk);
    float S = m.s0[(long long)sp * m.width + c];
    for (int j0 = 0; j0 < k; j0 += MG_UNROLL)
    {
        float av[MG_UNROLL], bv[MG_UNROLL];
        #pragma unroll
        for (int j = 0; j < MG_UNROLL; j++)
        {
            const long long at = (long long)(first + min(j0 + j, k - 1)) * m.width + c;
            av[j] = m.agg_a[at];
            bv[j] = m.agg_b[at];
        }
        #pragma unroll
        for (int j = 0; j < MG_UNROLL; j++)
            if (j0 + j < k) S = fmaf(av[j], S, bv[j]);
    }
    float a = 1.0f;
    S = mg_walk<T, true>(m, r0 + k * m.chunk, n, c, S, a);
    if ((k + 1) * m.chunk >= n_tok) m.state[(long long)m.row_seq[r0] * m.width + c] = S;
}

// ---- C ABI ----------------------------------------------------------------------------------------------------------------------

extern "C" int exl2_mingru_scan(const float* z, const float* u, const float* g, int ld, void* out, int ldo, float* state,
                                const int* span_row0, const int* span_rows, int spans, const int* row_seq, const int* row_pos,
                                const int* span_chunk0, int chunk, int total_chunks, float* scratch, int dtype, int width, void* stream)
{
    EXL2_REQUIRE(z && u && g && out && state && span_row0 && span_rows && row_seq && row_pos, "mingru_scan: null operand");
    EXL2_REQUIRE(dtype == 0 || dtype == 1, "mingru_scan: dtype must be 0 (bfloat16) or 1 (float32)");
    EXL2_REQUIRE(width > 0 && ld >= width && ldo >= width, "mingru_scan: bad shape");
    EXL2_REQUIRE(!scratch || (span_chunk0 && chunk > 0 && total_chunks > 0), "mingru_scan: the chunked form needs the chunk table");
    if (spans <= 0) return EXL2_OK;
    MinGruArgs m;
    m.z = z; m.u = u; m.g = g; m.ld = ld; m.out = out; m.ldo = ldo; m.state = state; m.span_row0 = span_row0; m.span_rows = span_rows;
    m.row_seq = row_seq; m.row_pos = row_pos; m.spans = spans; m.span_chunk0 = span_chunk0; m.chunk = chunk; m.width = width;
    m.agg_a = scratch; m.agg_b = scratch ? scratch + (long long)total_chunks * width : nullptr;
    m.s0 = scratch ? scratch + 2ll * total_chunks * width : nullptr;
    const int cb = (width + 255) / 256;
    if (!scratch)
    {
        if (dtype == 0) LAUNCH(mingru_kernel<u16>, dim3(cb, spans), dim3(256), 0, stream, m);
        else LAUNCH(mingru_kernel<float>, dim3(cb, spans), dim3(256), 0, stream, m);
    }
    else if (dtype == 0)
    {
        LAUNCH(mingru_chunk_kernel<u16>, dim3(cb, total_chunks), dim3(256), 0, stream, m);
        LAUNCH(mingru_out_kernel<u16>, dim3(cb, total_chunks), dim3(256), 0, stream, m);
    }
    else
    {
        LAUNCH(mingru_chunk_kernel<float>, dim3(cb, total_chunks), dim3(256), 0, stream, m);
        LAUNCH(mingru_out_kernel<float>, dim3(cb, total_chunks), dim3(256), 0, stream, m);
    }
    HIP_TRY(hipGetLastError());
    return EXL2_OK;
}
