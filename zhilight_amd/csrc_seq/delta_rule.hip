// delta_rule.hip -- the gated delta rule over a ragged step: a matrix memory S per head that decays, is read at the token's key, corrected
// towards the token's value and read at the token's query.
//
// k_delta_prep  everything a token needs before the recurrence, in one launch: the causal short convolution + SiLU on q, k and v (the
//               carried tail moves on), unit vectors per query / key head, the product q . k, beta, the decay per head or key channel.  A wave
//               per unit of work -- a query head with its key head (lanes over the coordinates), 256 value channels, 256 decays, the betas --
//               and block of consecutive tokens: the convolution's inputs slide through registers.
// k_delta_scan  a workgroup per (sequence, head, group of value columns).  Columns of S never meet, so every column walks the tokens on its
//               own: NGL neighbouring lanes hold a column, NPT numbers each, and meet in two DPP butterflies per token.  With a = g S the
//               token needs only the sums a.k and a.q at once:  u = beta (v - a.k),  S = a + k u,  o = a.q + (q.k) u.
//               The state lies (head, column, key coordinate), so a lane's numbers are 16-byte runs.
// k_delta_step  the same for a step of single tokens, without staging
// All of it is fp32 in both serving formats.
#include "seq_common.h"

namespace {

constexpr int kMaxR = 8;             // coordinates of a query / key head per lane in k_delta_prep: dim <= 64 * kMaxR

struct PrepP {
    const float* proj; int64_t ld; int col0;                 // [q (kv_heads * dim) | k (kv_heads * dim) | v (heads * vdim)] of a projection row
    const float* w; float* tail; int taps;                   // (channels, taps); (slots, taps - 1, channels)
    int heads, kv_heads, dim, vdim;
    float q_scale, unit_eps;
    int b_col0;                                              // beta's columns of the same rows
    const float* z; int64_t ldz; int z_col0;                 // what the decay is computed from: heads numbers per token, or heads * dim
    const float* z_bias; const float* rate;                  // z_bias nullable, one per number of z; rate (heads): g = exp(-rate softplus(z + z_bias))
    int per_channel;
    float* qkv; float* gates; float* decay;                  // gates (n_tok, heads, 4) = beta, decay per head (or 1), q . k, 0
    int n_tok, block;                                        // tokens per workgroup
};

// R channels of a lane, 64 apart: their convolution weights and the inputs of the last TAPS tokens in registers (TAPS 0: any number of taps,
// nothing kept)
template <int TAPS, int R>
struct ConvLane {
    float w[R][TAPS > 0 ? TAPS : 1], x[R][TAPS > 0 ? TAPS : 1];
    const PrepP& p; const float* row0; float* tl; int C, c0, lane, n, have;      // have: the token whose window x holds (-1: none)
    __device__ __forceinline__ ConvLane(const PrepP& p_, int C_, int c0_, int lane_, int n_) : p(p_), C(C_), c0(c0_), lane(lane_), n(n_), have(-1) {
        row0 = nullptr; tl = nullptr;
        if constexpr (TAPS > 0)
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
                for (int j = 0; j < TAPS; ++j) w[r][j] = ok(r) ? p.w[(size_t)(c0 + lane + 64 * r) * TAPS + j] : 0.f;
    }
    __device__ __forceinline__ bool ok(int r) const { return 64 * r < n && lane + 64 * r < n; }
    // the portion (its first projection row) that the following tokens belong to
    __device__ __forceinline__ void sequence(const float* row0_, float* tl_) {
        if (row0_ != row0) have = -1;
        row0 = row0_; tl = tl_;
    }
    __device__ __forceinline__ float input(int i, int r) const {                 // token i of the portion; i = -1 is the newest tail row
        const int c = c0 + lane + 64 * r;
        return i >= 0 ? row0[(size_t)i * p.ld + p.col0 + c] : tl[(size_t)(p.taps - 1 + i) * C + c];
    }
    // silu(convolution) at token i of the portion
    __device__ __forceinline__ void at(int i, float* out) {
        if constexpr (TAPS > 0) {
            if (have == i - 1 && i > 0) {
#pragma unroll
                for (int r = 0; r < R; ++r) {
#pragma unroll
                    for (int j = 0; j + 1 < TAPS; ++j) x[r][j] = x[r][j + 1];
                    x[r][TAPS - 1] = ok(r) ? input(i, r) : 0.f;
                }
            } else {
#pragma unroll
                for (int r = 0; r < R; ++r)
#pragma unroll
                    for (int j = 0; j < TAPS; ++j) x[r][j] = ok(r) ? input(i - (TAPS - 1 - j), r) : 0.f;
            }
            have = i;
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float a = 0.f;
#pragma unroll
                for (int j = 0; j < TAPS; ++j) a = fmaf(w[r][j], x[r][j], a);
                out[r] = seq_silu(a);
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float a = 0.f;
                if (ok(r))
                    for (int j = 0; j < p.taps; ++j) a = fmaf(p.w[(size_t)(c0 + lane + 64 * r) * p.taps + j], input(i - (p.taps - 1 - j), r), a);
                out[r] = seq_silu(a);
            }
        }
    }
    // the portion's last taps - 1 inputs become the tail (a lane owns its channels; rows in increasing order, each read before it is overwritten)
    __device__ __forceinline__ void shift(int count) {
        if (TAPS > 0 && count == 1) {                                            // (a single token's window holds them already)
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
                for (int j = 0; j + 1 < TAPS; ++j)
                    if (ok(r)) tl[(size_t)j * C + c0 + lane + 64 * r] = x[r][j + 1];
            return;
        }
#pragma unroll
        for (int r = 0; r < R; ++r)
            if (ok(r))
                for (int j = 0; j < p.taps - 1; ++j) tl[(size_t)j * C + c0 + lane + 64 * r] = input(count - (p.taps - 1) + j, r);
    }
};

template <int TAPS, int R>               // R: 64-coordinate parts of a query / key head
__global__ __launch_bounds__(256) void k_delta_prep(const PrepP p, const zls_batch_t b) {
    const int lane = threadIdx.x & 63, taps = p.taps;
    const int G = p.kv_heads, d = p.dim, V = p.heads * p.vdim, C = 2 * G * d + V, D = p.per_channel ? p.heads * d : p.heads, per = p.heads / G;
    const int nv = (V + 255) / 256, nd = p.per_channel ? (D + 255) / 256 : 0, units = G + nv + nd + 1;
    const int t_beg = blockIdx.x * p.block, t_end = min(p.n_tok, t_beg + p.block);
    // calls f(first flat token, portion length, token inside the portion, tail) for the tokens of this block
    auto tokens = [&](auto&& f) {
        for (int t = t_beg; t < t_end; ++t) {
            const int sq = b.tok_seq[t], first = b.seq_start[sq];
            f(first, b.seq_start[sq + 1] - first, t - first, p.tail + (size_t)b.seq_slot[sq] * (taps - 1) * C);
        }
    };
    // The block of a portion's first token convolves its tokens up to taps - 2 -- the only ones that look into the carried tail -- and then
    // moves the tail on; nobody else does those
    for (int u = blockIdx.y * 4 + (threadIdx.x >> 6); u < units; u += gridDim.y * 4) {
        if (u < G) {
            ConvLane<TAPS, R> cq(p, C, u * d, lane, d), ck(p, C, (G + u) * d, lane, d);
            tokens([&](int first, int count, int i0, float* tl) {
                if (i0 > 0 && i0 < taps - 1) return;
                cq.sequence(p.proj + (size_t)first * p.ld, tl);
                ck.sequence(p.proj + (size_t)first * p.ld, tl);
                const int n = i0 == 0 ? max(1, min(count, taps - 1)) : 1;
                for (int i = i0; i < i0 + n; ++i) {
                    float q[R], k[R], sq2 = 0.f, sk2 = 0.f, dot = 0.f;
                    cq.at(i, q);
                    ck.at(i, k);
#pragma unroll
                    for (int r = 0; r < R; ++r) {
                        sq2 = fmaf(q[r], q[r], sq2);
                        sk2 = fmaf(k[r], k[r], sk2);
                        dot = fmaf(q[r], k[r], dot);
                    }
#pragma unroll
                    for (int off = 32; off > 0; off >>= 1) {     // (three butterflies side by side)
                        sq2 += __shfl_xor(sq2, off, 64);
                        sk2 += __shfl_xor(sk2, off, 64);
                        dot += __shfl_xor(dot, off, 64);
                    }
                    const float fq = p.q_scale / sqrtf(sq2 + p.unit_eps), fk = 1.0f / sqrtf(sk2 + p.unit_eps);
                    float* row = p.qkv + (size_t)(first + i) * C + u * d;
#pragma unroll
                    for (int r = 0; r < R; ++r)
                        if (cq.ok(r)) {
                            row[lane + 64 * r] = q[r] * fq;
                            row[G * d + lane + 64 * r] = k[r] * fk;
                        }
                    for (int e = lane; e < per; e += 64) p.gates[((size_t)(first + i) * p.heads + u * per + e) * 4 + 2] = dot * fq * fk;
                }
                if (i0 == 0) { cq.shift(count); ck.shift(count); }
            });
        } else if (u < G + nv) {
            const int c0 = 2 * G * d + (u - G) * 256;
            ConvLane<TAPS, 4> cv(p, C, c0, lane, min(256, C - c0));
            tokens([&](int first, int count, int i0, float* tl) {
                if (i0 > 0 && i0 < taps - 1) return;
                cv.sequence(p.proj + (size_t)first * p.ld, tl);
                const int n = i0 == 0 ? max(1, min(count, taps - 1)) : 1;
                for (int i = i0; i < i0 + n; ++i) {
                    float v[4];
                    cv.at(i, v);
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (cv.ok(r)) p.qkv[(size_t)(first + i) * C + c0 + lane + 64 * r] = v[r];
                }
                if (i0 == 0) cv.shift(count);
            });
        } else if (u < G + nv + nd) {
            float zb[4], rt[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = min((u - G - nv) * 256 + r * 64 + lane, D - 1);
                zb[r] = p.z_bias ? p.z_bias[e] : 0.f;
                rt[r] = p.rate[e / d];
            }
            for (int t = t_beg; t < t_end; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int e = (u - G - nv) * 256 + r * 64 + lane;
                    if (e < D) p.decay[(size_t)t * D + e] = expf(-rt[r] * seq_softplus(p.z[(size_t)t * p.ldz + p.z_col0 + e] + zb[r]));
                }
        } else {
            for (int t = t_beg; t < t_end; ++t)
                for (int h = lane; h < p.heads; h += 64) {
                    float* g = p.gates + ((size_t)t * p.heads + h) * 4;
                    g[0] = seq_sigmoid(p.proj[(size_t)t * p.ld + p.b_col0 + h]);
                    g[1] = p.per_channel ? 1.0f
                                         : expf(-p.rate[h] * seq_softplus(p.z[(size_t)t * p.ldz + p.z_col0 + h] + (p.z_bias ? p.z_bias[h] : 0.f)));
                    g[3] = 0.f;
                }
        }
    }
}

struct DeltaP {
    const float* qkv; const float* gates; const float* decay;
    float* state; float* y;
    int heads, kv_heads, dim, vdim, vec;                      // vec: rows of q, k, decay and state in 16-byte pieces
};

template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
    return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// every lane plus the lane 16 / 32 further on: the swap instructions exchange odd rows (upper halves) of one register with even rows (lower
// halves) of the other, so two copies of v come out as the two addends
__device__ __forceinline__ float rows_add(float v) {
    const auto r = __builtin_amdgcn_permlane16_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    return __builtin_bit_cast(float, (uint32_t)r[0]) + __builtin_bit_cast(float, (uint32_t)r[1]);
}
__device__ __forceinline__ float halves_add(float v) {
    const auto r = __builtin_amdgcn_permlane32_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    return __builtin_bit_cast(float, (uint32_t)r[0]) + __builtin_bit_cast(float, (uint32_t)r[1]);
}
// two sums over NGL neighbouring lanes, in every lane: quads by permutation (xor 1, xor 2), then mirrored halves and rows of 16
template <int NGL>
__device__ __forceinline__ void group_sums(float& a, float& b) {
    a = dpp_add<0xB1>(a); b = dpp_add<0xB1>(b);
    a = dpp_add<0x4E>(a); b = dpp_add<0x4E>(b);
    if constexpr (NGL >= 8) { a = dpp_add<0x141>(a); b = dpp_add<0x141>(b); }
    if constexpr (NGL >= 16) { a = dpp_add<0x140>(a); b = dpp_add<0x140>(b); }
    if constexpr (NGL >= 32) { a = rows_add(a); b = rows_add(b); }
    if constexpr (NGL >= 64) { a = halves_add(a); b = halves_add(b); }
}

__device__ __forceinline__ float4 load4(const float* p, int n, int vec) {      // up to 4 numbers, n of them there
    if (vec) return *reinterpret_cast<const float4*>(p);
    return make_float4(p[0], n > 1 ? p[1] : 0.f, n > 2 ? p[2] : 0.f, n > 3 ? p[3] : 0.f);
}

constexpr int kScanT = 128;                                   // threads of a scan workgroup

// NGL lanes per column, NPT numbers per lane (coordinates 4 (g + NGL i) + e), CPL columns per group of lanes, PC: a decay per key channel.
// The tokens go through two LDS buffers of CH tokens, each four runs of rows: [k | q], decays (PC), the values of the workgroup's columns,
// [beta, decay, q.k, 0].  The next chunk's loads are in flight while the current one is walked; a token's rows are read into registers one
// token ahead.  At one wave per SIMD every instruction of the walk costs its four cycles, so a full chunk is unrolled: its addresses are
// immediates, and lane g of a column keeps the output of every NGL-th token, so that NGL tokens leave in one store.
template <int NGL, int NPT, int CPL, bool PC>
__global__ __launch_bounds__(kScanT) void k_delta_scan(const DeltaP p, const zls_batch_t b) {
    constexpr int F = NPT / 4, DP = NGL * NPT, D4 = DP / 4, CH = DP <= 128 ? 16 : DP == 256 ? 8 : 4, GROUPS = kScanT / NGL, COLS = GROUPS * CPL;
    constexpr int GO = (CH + 1) * 2 * DP, VO = GO + (PC ? (CH + 1) * DP : 0), SO = VO + ((CH + 1) * COLS + 3) / 4 * 4, BUF = SO + (CH + 1) * 4;
    constexpr int NK = (CH * 2 * D4 + kScanT - 1) / kScanT, NG = (CH * D4 + kScanT - 1) / kScanT, NV = (CH * COLS + kScanT - 1) / kScanT;
    static_assert(kScanT % D4 == 0 && 2 * BUF * sizeof(float) <= 64 * 1024, "a thread's pieces share their place in the row; two buffers");
    __shared__ __attribute__((aligned(16))) float lds[2 * BUF];              // (a row more in every run: the walk reads a token ahead)
    const int tid = threadIdx.x, g = tid % NGL, ci = tid / NGL;
    const int sq = blockIdx.x, h = blockIdx.y, hk = h / (p.heads / p.kv_heads), p0 = blockIdx.z * COLS;
    const int d = p.dim, P = p.vdim, H = p.heads;
    const int first = b.seq_start[sq], count = b.seq_start[sq + 1] - first;
    const int qk_dim = p.kv_heads * d, C = 2 * qk_dim + H * P;
    float* st = p.state + ((size_t)b.seq_slot[sq] * H + h) * P * d;
    float S[CPL][NPT];
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int col = p0 + ci + c * GROUPS;
#pragma unroll
        for (int i = 0; i < F; ++i) {
            const int n = 4 * (g + NGL * i);
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (col < P && n < d) v = load4(st + (size_t)col * d + n, d - n, p.vec);
            S[c][4 * i] = v.x; S[c][4 * i + 1] = v.y; S[c][4 * i + 2] = v.z; S[c][4 * i + 3] = v.w;
        }
    }
    if (d < DP || P % COLS)                                  // what no token writes -- coordinates past dim, columns past vdim -- is 0 for good
        for (int i = tid; i < 2 * BUF; i += kScanT) lds[i] = 0.f;

    // the next chunk in registers: piece tid + kScanT u of a run
    float4 kr[NK], gr[PC ? NG : 1], sr;
    float vr[NV];
    const int f = tid % D4;
    const bool fok = 4 * f < d;
    auto fetch = [&](int c0) {
        const int cn = min(CH, count - c0);
        const float* rows = p.qkv + (size_t)(first + c0) * C;
        const float* dec = PC ? p.decay + ((size_t)(first + c0) * H + h) * d : nullptr;
        auto pieces = [&](auto full, int vec) {
#pragma unroll
            for (int u = 0; u < NK; ++u) {
                const int rr = (u * kScanT + tid) / D4, run = rr & 1, i = rr >> 1;
                if ((full && CH * 2 * D4 % kScanT == 0) || i < cn)
                    if (fok) kr[u] = load4(rows + i * C + (run ? 0 : qk_dim) + hk * d + 4 * f, d - 4 * f, vec);
            }
            if constexpr (PC) {
#pragma unroll
                for (int u = 0; u < NG; ++u) {
                    const int i = (u * kScanT + tid) / D4;
                    if ((full && CH * D4 % kScanT == 0) || i < cn)
                        if (fok) gr[u] = load4(dec + i * H * d + 4 * f, d - 4 * f, vec);
                }
            }
        };
        if (!p.vec) pieces(false, 0);
        else if (cn == CH) pieces(true, 1);
        else pieces(false, 1);
#pragma unroll
        for (int u = 0; u < NV; ++u) {
            const int e = u * kScanT + tid, i = e / COLS, c = e % COLS;
            if (i < cn && p0 + c < P) vr[u] = rows[i * C + 2 * qk_dim + h * P + p0 + c];
        }
        if (tid < cn) sr = *reinterpret_cast<const float4*>(p.gates + ((size_t)(first + c0 + tid) * H + h) * 4);
    };
    auto publish = [&](int c0, float* dst) {
        const int cn = min(CH, count - c0);
#pragma unroll
        for (int u = 0; u < NK; ++u) {
            const int e = u * kScanT + tid;
            if (fok && e < cn * 2 * D4) *reinterpret_cast<float4*>(dst + 4 * e) = kr[u];
        }
        if constexpr (PC) {
#pragma unroll
            for (int u = 0; u < NG; ++u) {
                const int e = u * kScanT + tid;
                if (fok && e < cn * D4) *reinterpret_cast<float4*>(dst + GO + 4 * e) = gr[u];
            }
        }
#pragma unroll
        for (int u = 0; u < NV; ++u) {
            const int e = u * kScanT + tid;
            if (e < cn * COLS && p0 + e % COLS < P) dst[VO + e] = vr[u];
        }
        if (tid < cn) *reinterpret_cast<float4*>(dst + SO + 4 * tid) = sr;
    };

    fetch(0);
    __builtin_amdgcn_s_waitcnt(0x0F70);                      // vmcnt(0): the state's numbers are here (the walk's loop must not wait for them)
    __syncthreads();
    publish(0, lds);
    __syncthreads();
    float* yc[CPL];                                          // the column of the chunk's first token
#pragma unroll
    for (int c = 0; c < CPL; ++c) yc[c] = p.y + ((size_t)first * H + h) * P + min(p0 + ci + c * GROUPS, P - 1);
    const int ystep = H * P;
    struct Row { float4 k[F], q[F], g[F], sc; float v[CPL]; };
    for (int c0 = 0, which = 0; c0 < count; c0 += CH, which ^= 1) {
        const int cn = min(CH, count - c0);
        const bool more = c0 + CH < count;
        if (more) fetch(c0 + CH);                            // in flight during the walk
        const float* base = lds + which * BUF + 4 * g;
        const float* vbase = lds + which * BUF + VO + ci;
        const float* sbase = lds + which * BUF + SO;
        auto read = [&](Row& r, int i) {
#pragma unroll
            for (int f = 0; f < F; ++f) {
                r.k[f] = *reinterpret_cast<const float4*>(base + i * 2 * DP + 4 * NGL * f);
                r.q[f] = *reinterpret_cast<const float4*>(base + i * 2 * DP + DP + 4 * NGL * f);
                if constexpr (PC) r.g[f] = *reinterpret_cast<const float4*>(base + GO + i * DP + 4 * NGL * f);
            }
            r.sc = *reinterpret_cast<const float4*>(sbase + 4 * i);
#pragma unroll
            for (int c = 0; c < CPL; ++c) r.v[c] = vbase[i * COLS + c * GROUPS];
        };
        float keep[CPL];
        auto step = [&](const Row& r, int i) {
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
                float dk, dq;
#pragma unroll
                for (int f = 0; f < F; ++f) {
                    const float4 gg = PC ? r.g[f] : make_float4(r.sc.y, r.sc.y, r.sc.y, r.sc.y);
                    float* s = S[c] + 4 * f;
                    s[0] *= gg.x; s[1] *= gg.y; s[2] *= gg.z; s[3] *= gg.w;
                    if (f == 0) { dk = s[0] * r.k[f].x; dq = s[0] * r.q[f].x; }
                    else { dk = fmaf(s[0], r.k[f].x, dk); dq = fmaf(s[0], r.q[f].x, dq); }
                    dk = fmaf(s[1], r.k[f].y, dk); dq = fmaf(s[1], r.q[f].y, dq);
                    dk = fmaf(s[2], r.k[f].z, dk); dq = fmaf(s[2], r.q[f].z, dq);
                    dk = fmaf(s[3], r.k[f].w, dk); dq = fmaf(s[3], r.q[f].w, dq);
                }
                group_sums<NGL>(dk, dq);
                const float u = r.sc.x * (r.v[c] - dk);
#pragma unroll
                for (int f = 0; f < F; ++f) {
                    float* s = S[c] + 4 * f;
                    s[0] = fmaf(r.k[f].x, u, s[0]); s[1] = fmaf(r.k[f].y, u, s[1]); s[2] = fmaf(r.k[f].z, u, s[2]); s[3] = fmaf(r.k[f].w, u, s[3]);
                }
                const float o = fmaf(r.sc.z, u, dq);
                keep[c] = g == (i & (NGL - 1)) ? o : keep[c];
            }
        };
        auto store = [&](int i) {                            // the outputs of the tokens (i rounded down to NGL) .. i
            const int j = (i & ~(NGL - 1)) + g;
#pragma unroll
            for (int c = 0; c < CPL; ++c)
                if (j <= i && p0 + ci + c * GROUPS < P) yc[c][j * ystep] = keep[c];
        };
        Row r0, r1;
#pragma unroll
        for (int c = 0; c < CPL; ++c) keep[c] = 0.f;
        read(r0, 0);
        if (cn == CH) {
#pragma unroll
            for (int i = 0; i < CH; i += 2) {
                read(r1, i + 1);
                __builtin_amdgcn_sched_barrier(0);           // (the reads go out before the token's arithmetic, not between its last steps)
                step(r0, i);
                if (((i + 1) & (NGL - 1)) == 0) store(i);
                read(r0, i + 2);
                __builtin_amdgcn_sched_barrier(0);
                step(r1, i + 1);
                if (((i + 2) & (NGL - 1)) == 0 || i + 2 == CH) store(i + 1);
            }
        } else {
            for (int i = 0; i < cn; ++i) {
                step(r0, i);
                if (((i + 1) & (NGL - 1)) == 0 || i + 1 == cn) store(i);
                read(r0, i + 1);
            }
        }
#pragma unroll
        for (int c = 0; c < CPL; ++c) yc[c] += (size_t)CH * ystep;
        if (more) publish(c0 + CH, lds + (which ^ 1) * BUF); // (the chunk that buffer held was walked before the last barrier)
        __syncthreads();
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
        const int col = p0 + ci + c * GROUPS;
#pragma unroll
        for (int i = 0; i < F; ++i) {
            const int n = 4 * (g + NGL * i);
            if (col >= P || n >= d) continue;
            float* o = st + (size_t)col * d + n;
            if (p.vec) {
                *reinterpret_cast<float4*>(o) = make_float4(S[c][4 * i], S[c][4 * i + 1], S[c][4 * i + 2], S[c][4 * i + 3]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < d) o[e] = S[c][4 * i + e];
            }
        }
    }
}

// A step in which every portion is ONE token: the state is the traffic.  Nothing is staged -- a lane reads its numbers of the state, the
// token's key, query and decays straight from memory, all loads in flight together, and writes its numbers of the state back.
template <int NGL, int NPT, bool PC>
__global__ __launch_bounds__(256) void k_delta_step(const DeltaP p, const zls_batch_t b) {
    constexpr int F = NPT / 4;
    const int g = threadIdx.x % NGL, sq = blockIdx.x, h = blockIdx.y, hk = h / (p.heads / p.kv_heads), col = blockIdx.z * (256 / NGL) + threadIdx.x / NGL;
    const int d = p.dim, P = p.vdim, H = p.heads, qk_dim = p.kv_heads * d, C = 2 * qk_dim + H * P;
    const size_t t = b.seq_start[sq];
    const bool ok = col < P;
    float* st = p.state + (((size_t)b.seq_slot[sq] * H + h) * P + (ok ? col : 0)) * d;
    const float* row = p.qkv + t * C + hk * d;
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 s[F], k[F], q[F], a[F];
    const float4 sc = *reinterpret_cast<const float4*>(p.gates + (t * H + h) * 4);
#pragma unroll
    for (int f = 0; f < F; ++f) {
        const int n = 4 * (g + NGL * f);
        s[f] = k[f] = q[f] = zero;
        a[f] = make_float4(sc.y, sc.y, sc.y, sc.y);
        if (n < d) {
            s[f] = load4(st + n, d - n, p.vec);
            k[f] = load4(row + qk_dim + n, d - n, p.vec);
            q[f] = load4(row + n, d - n, p.vec);
            if constexpr (PC) a[f] = load4(p.decay + (t * H + h) * d + n, d - n, p.vec);
        }
    }
    const float v = ok ? p.qkv[t * C + 2 * qk_dim + h * P + col] : 0.f;
    float dk = 0.f, dq = 0.f;
#pragma unroll
    for (int f = 0; f < F; ++f) {
        s[f].x *= a[f].x; s[f].y *= a[f].y; s[f].z *= a[f].z; s[f].w *= a[f].w;
        dk = fmaf(s[f].x, k[f].x, dk); dk = fmaf(s[f].y, k[f].y, dk); dk = fmaf(s[f].z, k[f].z, dk); dk = fmaf(s[f].w, k[f].w, dk);
        dq = fmaf(s[f].x, q[f].x, dq); dq = fmaf(s[f].y, q[f].y, dq); dq = fmaf(s[f].z, q[f].z, dq); dq = fmaf(s[f].w, q[f].w, dq);
    }
    group_sums<NGL>(dk, dq);
    const float u = sc.x * (v - dk);
    if (!ok) return;
    if (g == 0) p.y[(t * H + h) * P + col] = fmaf(sc.z, u, dq);
#pragma unroll
    for (int f = 0; f < F; ++f) {
        const int n = 4 * (g + NGL * f);
        if (n >= d) continue;
        const float r[4] = {fmaf(k[f].x, u, s[f].x), fmaf(k[f].y, u, s[f].y), fmaf(k[f].z, u, s[f].z), fmaf(k[f].w, u, s[f].w)};
        if (p.vec) {
            *reinterpret_cast<float4*>(st + n) = make_float4(r[0], r[1], r[2], r[3]);
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (n + e < d) st[n + e] = r[e];
        }
    }
}

}  // namespace

extern "C" int zls_delta_prep(const float* proj, int64_t ld, int64_t col0, const float* w, float* tail, int64_t taps, int64_t heads, int64_t kv_heads,
                              int64_t dim, int64_t vdim, float q_scale, float unit_eps, int64_t b_col0, const float* z, int64_t ldz, int64_t z_col0,
                              const float* z_bias, const float* rate, int per_channel, const zls_batch_t* b, float* qkv, float* gates, float* decay,
                              zl_stream_t s) {
    ZL_CHECK_ARG(proj && w && z && rate && qkv && gates && (decay || !per_channel) && seq_batch_ok(b) && taps > 0 && (tail || taps == 1), ZL_EINVAL);
    ZL_CHECK_ARG(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, ZL_ESHAPE);
    const int64_t C = 2 * kv_heads * dim + heads * vdim, D = per_channel ? heads * dim : heads;
    ZL_CHECK_ARG(col0 >= 0 && col0 + C <= ld && b_col0 >= 0 && b_col0 + heads <= ld && z_col0 >= 0 && z_col0 + D <= ldz, ZL_ESHAPE);
    ZL_CHECK_ARG(dim <= 64 * kMaxR && C < (1 << 28) && D < (1 << 28) && taps < (1 << 16), ZL_ELIMIT);
    PrepP p = {};
    p.proj = proj; p.ld = ld; p.col0 = (int)col0; p.w = w; p.tail = tail; p.taps = (int)taps; p.heads = (int)heads; p.kv_heads = (int)kv_heads;
    p.dim = (int)dim; p.vdim = (int)vdim; p.q_scale = q_scale; p.unit_eps = unit_eps; p.b_col0 = (int)b_col0; p.z = z; p.ldz = ldz;
    p.z_col0 = (int)z_col0; p.z_bias = z_bias; p.rate = rate; p.per_channel = per_channel ? 1 : 0; p.qkv = qkv; p.gates = gates; p.decay = decay;
    const int64_t units = kv_heads + (heads * vdim + 255) / 256 + (per_channel ? (D + 255) / 256 : 0) + 1, want = (units + 3) / 4;
    p.n_tok = b->n_tok;
    p.block = b->n_tok * want >= 4096 ? 8 : b->n_tok * want >= 2048 ? 4 : 1;     // (a block of tokens per workgroup when they fill the chip all the same)
    const dim3 grid((unsigned)((b->n_tok + p.block - 1) / p.block), (unsigned)(want < 1024 ? want : 1024));
#define GO(TAPS, R) hipLaunchKernelGGL((k_delta_prep<TAPS, R>), grid, dim3(256), 0, (hipStream_t)s, p, *b)
#define HEAD(TAPS)                                          \
    if (dim <= 64) GO(TAPS, 1);                             \
    else if (dim <= 128) GO(TAPS, 2);                       \
    else if (dim <= 256) GO(TAPS, 4);                       \
    else GO(TAPS, 8)
    if (taps == 2) { HEAD(2); }
    else if (taps == 3) { HEAD(3); }
    else if (taps == 4) { HEAD(4); }
    else { HEAD(0); }
#undef HEAD
#undef GO
    return zl_launch_status();
}

extern "C" int zls_delta_scan(const float* qkv, const float* gates, const float* decay, float* state, int64_t heads, int64_t kv_heads, int64_t dim,
                              int64_t vdim, const zls_batch_t* b, float* y, zl_stream_t s) {
    ZL_CHECK_ARG(qkv && gates && state && y && seq_batch_ok(b), ZL_EINVAL);
    ZL_CHECK_ARG(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0, ZL_ESHAPE);
    const int64_t C = 2 * kv_heads * dim + heads * vdim;
    auto al = [](const void* q) { return ((uintptr_t)q & 15) == 0; };
    ZL_CHECK_ARG(dim <= 512 && vdim <= (1 << 20) && C * 64 < (1LL << 31) && heads * dim * 64 < (1LL << 31) && al(gates), ZL_ELIMIT);
    DeltaP p = {};
    p.qkv = qkv; p.gates = gates; p.decay = decay; p.state = state; p.y = y; p.heads = (int)heads; p.kv_heads = (int)kv_heads;
    p.dim = (int)dim; p.vdim = (int)vdim;
    p.vec = (dim % 4 == 0 && C % 4 == 0 && al(qkv) && al(state) && (!decay || al(decay))) ? 1 : 0;
    const int ngl = dim <= 16 ? 4 : dim <= 32 ? 8 : dim <= 128 ? 16 : dim <= 256 ? 32 : 64;
    hipStream_t hs = (hipStream_t)s;
    if (b->max_count == 1) {
        const int64_t parts = (vdim * ngl + 255) / 256;
        ZL_CHECK_ARG(parts <= 65535, ZL_ELIMIT);
        const dim3 grid((unsigned)b->n_seq, (unsigned)heads, (unsigned)parts);
#define STEP(NGL, NPT)                                                                                         \
    if (decay) hipLaunchKernelGGL((k_delta_step<NGL, NPT, true>), grid, dim3(256), 0, hs, p, *b);              \
    else hipLaunchKernelGGL((k_delta_step<NGL, NPT, false>), grid, dim3(256), 0, hs, p, *b)
        if (dim <= 16) { STEP(4, 4); }
        else if (dim <= 32) { STEP(8, 4); }
        else if (dim <= 64) { STEP(16, 4); }
        else if (dim <= 128) { STEP(16, 8); }
        else if (dim <= 256) { STEP(32, 8); }
        else { STEP(64, 8); }
#undef STEP
        return zl_launch_status();
    }
    // two columns per group of lanes once single ones fill the chip's 1024 SIMDs
    const int64_t waves = (int64_t)b->n_seq * heads * ((vdim * ngl + 63) / 64);
    const int cpl = waves > 1024 && vdim * ngl > kScanT ? 2 : 1, cols = kScanT / ngl * cpl;
    const int64_t parts = (vdim + cols - 1) / cols;
    ZL_CHECK_ARG(parts <= 65535 && heads * vdim * 64 < (1LL << 31), ZL_ELIMIT);
    const dim3 grid((unsigned)b->n_seq, (unsigned)heads, (unsigned)parts);
#define GO(NGL, NPT, CPL, PC) hipLaunchKernelGGL((k_delta_scan<NGL, NPT, CPL, PC>), grid, dim3(kScanT), 0, hs, p, *b)
#define SIZES(NGL, NPT)                                                                 \
    if (cpl == 2) { if (decay) GO(NGL, NPT, 2, true); else GO(NGL, NPT, 2, false); }    \
    else { if (decay) GO(NGL, NPT, 1, true); else GO(NGL, NPT, 1, false); }
    if (dim <= 16) { SIZES(4, 4) }
    else if (dim <= 32) { SIZES(8, 4) }
    else if (dim <= 64) { SIZES(16, 4) }
    else if (dim <= 128) { SIZES(16, 8) }
    else if (dim <= 256) { SIZES(32, 8) }
    else { SIZES(64, 8) }
#undef SIZES
#undef GO
    return zl_launch_status();
}
