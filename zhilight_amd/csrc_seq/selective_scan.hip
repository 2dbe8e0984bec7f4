// selective_scan.hip -- the selective recurrence with a decay per channel AND state (Mamba) over a ragged step, its fp32 state carried per
// sequence slot:
//   S[n][c] <- 2^(dt_c a2[n][c]) S[n][c] + dt_c x_c B_n;   y_c = (sum_n S[n][c] C_n + d_c x_c) * silu(z_c)
//
// Unlike the scan of ssm.hip (one decay per head and token) every state has a decay of its own, an exponential per (token, channel, state): that is the
// work, and it has no matrix form.  What is shared is B and C: all channels of a token read the same n_state numbers.
//
// k_selective_scan<NPT>  a workgroup = 64 channels of one segment of one sequence; a lane owns a channel, a wave NPT of its states in
//                        registers (with their rates), `waves` waves all of them.  kTok tokens at a time: x and dt come straight into
//                        registers, one coalesced load per token (the next chunk's are requested before this chunk is walked), B and C go
//                        through LDS and are read back as broadcasts.  A wave leaves its part of y in LDS; after the next barrier the
//                        threads add the waves' parts, the skip term and the gate, and store the row in the serving format.  Both LDS areas
//                        alternate between two halves: one barrier per chunk.
// k_selective_combine    start states of the segments 1 .. of long portions.  A segment's decays multiply to 2^(a2 sum(dt)), so a segment
//                        only has to leave its end state from zero and its sum of dt.
// Long portions run as segments: mode 1 (end states from zero), combine, mode 2 (again, from the true start states, writing y).
#include "seq_common.h"

namespace {

constexpr int kTok = 8;                 // tokens per chunk
constexpr int kMaxWaves = 8;

struct SelP {
    const float* x; const float* dt; const float* bc; const float* zrow; const float* a2; const float* d;
    float* state; void* y;
    int64_t ldbc, ldz;
    int b_col0, c_col0, z_col0, inner, n_state, waves;
    int mode, seg_len, n_seg;           // 0: whole portions; 1: a segment's end state from zero; 2: a segment from its start state
    float* seg_state;                   // (n_seq, n_seg, n_state, inner): mode 1 leaves end states, k_selective_combine turns them into start states
    float* seg_dt;                      // (n_seq, n_seg, inner): sum of dt
};

template <int NPT, int DT>
__global__ __launch_bounds__(64 * kMaxWaves) void k_selective_scan(const SelP p, const zls_batch_t b) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nthr = blockDim.x;
    const int NP = p.waves * NPT;                                        // states padded to whole waves
    float* bcs = lds;                                                    // [2][kTok][2][NP]
    float* part = lds + 2 * kTok * 2 * NP;                               // [2][kTok][waves][64]
    const int sq = blockIdx.x / p.n_seg, seg = blockIdx.x % p.n_seg;
    const int whole = b.seq_start[sq + 1] - b.seq_start[sq];
    if (seg * p.seg_len >= whole) return;                                // (workgroup-uniform)
    const bool last_seg = (seg + 1) * p.seg_len >= whole;
    if (p.mode == 1 && last_seg) return;                                 // nobody starts from the last segment's end state
    const int first = b.seq_start[sq] + seg * p.seg_len, count = min(p.seg_len, whole - seg * p.seg_len);
    const int c = blockIdx.y * 64 + lane;
    const bool cok = c < p.inner;
    const int cl = cok ? c : p.inner - 1;                                // (lanes past the edge walk a copy of the last channel and store nothing)
    const int n0 = wave * NPT;
    float* st = p.state + (size_t)b.seq_slot[sq] * p.n_state * p.inner;
    const size_t seg_at = (size_t)sq * p.n_seg + seg;
    const float* init = (p.mode == 2 && seg > 0) ? p.seg_state + seg_at * p.n_state * p.inner : st;
    float S[NPT], A[NPT];
#pragma unroll
    for (int j = 0; j < NPT; ++j) {
        const bool ok = n0 + j < p.n_state;                              // (a padded state: rate 0, B = C = 0)
        A[j] = ok ? p.a2[(size_t)(n0 + j) * p.inner + cl] : 0.f;
        S[j] = (ok && p.mode != 1) ? init[(size_t)(n0 + j) * p.inner + cl] : 0.f;
    }
    // B and C of a chunk: kTok rows of 2 NP numbers, slot u of a thread = number tid + u * threads
    constexpr int kSlots = (kTok * 2 * NPT + 63) / 64;
    float pre[kSlots], px[kTok], pd[kTok];
    auto fetch = [&](int c0) {
        const int cn = min(kTok, count - c0);
#pragma unroll
        for (int u = 0; u < kSlots; ++u) {
            const int e = threadIdx.x + u * nthr, i = e / (2 * NP), r = e % (2 * NP), n = r % NP;
            pre[u] = (i < cn && n < p.n_state) ? p.bc[(size_t)(first + c0 + i) * p.ldbc + (r < NP ? p.b_col0 : p.c_col0) + n] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < kTok; ++i) {
            const size_t at = (size_t)(first + c0 + min(i, cn - 1)) * p.inner + cl;
            px[i] = p.x[at];
            pd[i] = p.dt[at];
        }
    };
    auto finish = [&](int c0, int half) {                                // the rows of chunk c0 from the waves' parts
        const int cn = min(kTok, count - c0);
        for (int i = wave; i < cn; i += p.waves) {
            const float* pt = part + ((half * kTok + i) * p.waves) * 64 + lane;
            float v = 0.f;
            for (int w = 0; w < p.waves; ++w) v += pt[w * 64];
            const size_t t = (size_t)(first + c0 + i);
            if (cok) SeqT<DT>::st(p.y, t * p.inner + c, fmaf(p.d[c], p.x[t * p.inner + c], v) * seq_silu(p.zrow[t * p.ldz + p.z_col0 + c]));
        }
    };
    float sum_dt = 0.f;
    fetch(0);
    int half = 0;
    for (int c0 = 0; c0 < count; c0 += kTok, half ^= 1) {
        const int cn = min(kTok, count - c0);
#pragma unroll
        for (int u = 0; u < kSlots; ++u) {
            const int e = threadIdx.x + u * nthr;
            if (e < kTok * 2 * NP) bcs[half * kTok * 2 * NP + e] = pre[u];
        }
        float xv[kTok], dv[kTok];
#pragma unroll
        for (int i = 0; i < kTok; ++i) { xv[i] = px[i]; dv[i] = i < cn ? pd[i] : 0.f; }
        __syncthreads();                                                 // this chunk's B / C and the previous chunk's parts are there
        if (c0 + kTok < count) fetch(c0 + kTok);
        if (p.mode != 1 && c0 > 0) finish(c0 - kTok, half ^ 1);
        // (tokens past the portion's end have dt = 0: decay 1, nothing added)
#pragma unroll
        for (int i = 0; i < kTok; ++i) {
            const float dt = dv[i], dx = dt * xv[i];
            const float4* Bv = reinterpret_cast<const float4*>(bcs + ((half * kTok + i) * 2) * NP + n0);
            const float4* Cv = reinterpret_cast<const float4*>(bcs + ((half * kTok + i) * 2 + 1) * NP + n0);
            float y0 = 0.f, y1 = 0.f;
            if (p.mode == 1) {
                sum_dt += dt;
#pragma unroll
                for (int j = 0; j < NPT; j += 4) {
                    const float4 bq = Bv[j >> 2];
                    S[j] = fmaf(__builtin_amdgcn_exp2f(dt * A[j]), S[j], bq.x * dx);
                    S[j + 1] = fmaf(__builtin_amdgcn_exp2f(dt * A[j + 1]), S[j + 1], bq.y * dx);
                    S[j + 2] = fmaf(__builtin_amdgcn_exp2f(dt * A[j + 2]), S[j + 2], bq.z * dx);
                    S[j + 3] = fmaf(__builtin_amdgcn_exp2f(dt * A[j + 3]), S[j + 3], bq.w * dx);
                }
                continue;
            }
#pragma unroll
            for (int j = 0; j < NPT; j += 4) {
                const float4 bq = Bv[j >> 2], cq = Cv[j >> 2];
                S[j] = fmaf(__builtin_amdgcn_exp2f(dt * A[j]), S[j], bq.x * dx);
                S[j + 1] = fmaf(__builtin_amdgcn_exp2f(dt * A[j + 1]), S[j + 1], bq.y * dx);
                S[j + 2] = fmaf(__builtin_amdgcn_exp2f(dt * A[j + 2]), S[j + 2], bq.z * dx);
                S[j + 3] = fmaf(__builtin_amdgcn_exp2f(dt * A[j + 3]), S[j + 3], bq.w * dx);
                y0 = fmaf(S[j], cq.x, y0);
                y1 = fmaf(S[j + 1], cq.y, y1);
                y0 = fmaf(S[j + 2], cq.z, y0);
                y1 = fmaf(S[j + 3], cq.w, y1);
            }
            part[((half * kTok + i) * p.waves + wave) * 64 + lane] = y0 + y1;
        }
    }
    if (p.mode != 1) {
        __syncthreads();
        finish((count - 1) / kTok * kTok, half ^ 1);
    }
    if (!cok || (p.mode == 2 && !last_seg)) return;                      // only the portion's last segment leaves the slot's state
    float* dst = p.mode == 1 ? p.seg_state + seg_at * p.n_state * p.inner : st;
#pragma unroll
    for (int j = 0; j < NPT; ++j)
        if (n0 + j < p.n_state) dst[(size_t)(n0 + j) * p.inner + c] = S[j];
    if (p.mode == 1 && wave == 0) p.seg_dt[seg_at * p.inner + c] = sum_dt;
}

// S_{k+1} = 2^(a2 sum of segment k's dt) S_k + (segment k's end state from zero), S_0 = the slot's state; segment k's entry of seg_state becomes
// S_k.  A thread per (state, channel), segments in order
__global__ __launch_bounds__(256) void k_selective_combine(const SelP p, const zls_batch_t b) {
    const int c = blockIdx.x * 256 + threadIdx.x, n = blockIdx.y, sq = blockIdx.z;
    if (c >= p.inner) return;
    const int whole = b.seq_start[sq + 1] - b.seq_start[sq];
    const int nseg = (whole + p.seg_len - 1) / p.seg_len;
    const size_t stride = (size_t)p.n_state * p.inner, at = (size_t)n * p.inner + c;
    float S = p.state[(size_t)b.seq_slot[sq] * stride + at];
    const float a = p.a2[at];
    for (int k = 0; k < nseg; ++k) {
        const size_t sk = (size_t)sq * p.n_seg + k;
        float* e = p.seg_state + sk * stride + at;
        const float next = k + 1 < nseg ? fmaf(__builtin_amdgcn_exp2f(a * p.seg_dt[sk * p.inner + c]), S, *e) : 0.f;
        *e = S;
        S = next;
    }
}

}  // namespace

extern "C" int64_t zls_selective_scan_workspace_bytes(int64_t n_seq, int64_t max_count, int64_t seg_len, int64_t inner, int64_t n_state) {
    if (n_seq <= 0 || max_count <= 0 || seg_len <= 0 || inner <= 0 || n_state <= 0) return ZL_EINVAL;
    const int64_t n_seg = (max_count + seg_len - 1) / seg_len;
    return n_seq * n_seg * inner * (n_state + 1) * (int64_t)sizeof(float);
}

extern "C" int zls_selective_scan(const float* x, const float* dt, const float* bc, int64_t ldbc, int64_t b_col0, int64_t c_col0, const float* zrow,
                                  int64_t ldz, int64_t z_col0, const float* a2, const float* d, float* state, int64_t inner, int64_t n_state,
                                  const zls_batch_t* b, void* y, void* workspace, int64_t seg_len, int dtype, zl_stream_t s) {
    ZL_CHECK_ARG(x && dt && bc && zrow && a2 && d && state && y && seq_batch_ok(b) && inner > 0 && n_state > 0, ZL_EINVAL);
    ZL_CHECK_ARG(b_col0 >= 0 && b_col0 + n_state <= ldbc && c_col0 >= 0 && c_col0 + n_state <= ldbc && z_col0 >= 0 && z_col0 + inner <= ldz, ZL_ESHAPE);
    ZL_CHECK_ARG(n_state <= 32 * kMaxWaves && inner <= 64 * 65535, ZL_ELIMIT);
    const bool segmented = workspace && seg_len > 0 && b->max_count > seg_len;
    const int64_t n_seg = segmented ? (b->max_count + seg_len - 1) / seg_len : 1;
    ZL_CHECK_ARG((int64_t)b->n_seq * n_seg <= 0x7fffffff && b->n_seq <= 65535, ZL_ELIMIT);
    const int npt = n_state <= 8 * kMaxWaves ? 8 : n_state <= 16 * kMaxWaves ? 16 : 32;
    SelP p = {};
    p.x = x; p.dt = dt; p.bc = bc; p.zrow = zrow; p.a2 = a2; p.d = d; p.state = state; p.y = y; p.ldbc = ldbc; p.ldz = ldz;
    p.b_col0 = (int)b_col0; p.c_col0 = (int)c_col0; p.z_col0 = (int)z_col0; p.inner = (int)inner; p.n_state = (int)n_state;
    p.waves = (int)((n_state + npt - 1) / npt);
    p.seg_len = segmented ? (int)seg_len : b->max_count;
    p.n_seg = (int)n_seg;
    p.seg_state = (float*)workspace;
    p.seg_dt = p.seg_state + (int64_t)b->n_seq * n_seg * inner * n_state;
    const size_t lds = (size_t)(2 * kTok * 2 * p.waves * npt + 2 * kTok * p.waves * 64) * sizeof(float);
    ZL_CHECK_ARG(lds <= 64 * 1024, ZL_ELIMIT);
    const dim3 grid((unsigned)(b->n_seq * n_seg), (unsigned)((inner + 63) / 64)), block((unsigned)(64 * p.waves));
    hipStream_t hs = (hipStream_t)s;
#define SCAN_N(DT, NPT) hipLaunchKernelGGL((k_selective_scan<NPT, DT>), grid, block, lds, hs, p, *b)
#define SCAN(DT)                                    \
    if (npt == 8) { SCAN_N(DT, 8); }                \
    else if (npt == 16) { SCAN_N(DT, 16); }         \
    else { SCAN_N(DT, 32); }
#define CALL(DT)                                                                                                                   \
    if (segmented) {                                                                                                               \
        p.mode = 1;                                                                                                                \
        SCAN(DT)                                                                                                                   \
        hipLaunchKernelGGL(k_selective_combine, dim3((unsigned)((inner + 255) / 256), (unsigned)n_state, (unsigned)b->n_seq), dim3(256), 0, hs, p, *b); \
        p.mode = 2;                                                                                                                \
    }                                                                                                                              \
    SCAN(DT)
    ZLS_DISPATCH(dtype, CALL)
#undef CALL
#undef SCAN
#undef SCAN_N
    return zl_launch_status();
}
