// A small JSON reader (RFC 8259) for model descriptions, safetensors headers and request traces: parses a whole text into a tree of
// values.  Malformed input throws JsonError with the byte position; so does asking a value for what it is not.
#pragma once

#include <cmath>
#include <cstdint>
#include <cstdlib>
#include <map>
#include <stdexcept>
#include <string>
#include <string_view>
#include <utility>
#include <vector>

namespace glint {

struct JsonError : std::runtime_error
{
  using std::runtime_error::runtime_error;
};

class Json
{
public:
  enum class Kind
  {
    Null,
    Bool,
    Number,
    String,
    Array,
    Object
  };

  static Json parse( const std::string_view text )
  {
    Parser p { text };
    Json v = p.value( 0 );
    p.space();
    if ( p.at != text.size() ) {
      p.fail( "text behind the value" );
    }
    return v;
  }

  Kind kind() const { return kind_; }
  bool is_null() const { return kind_ == Kind::Null; }

  double number() const
  {
    want( Kind::Number, "a number" );
    return number_;
  }
  // a whole number in [0, 2^53]
  uint64_t integer() const
  {
    const double d = number();
    if ( !( d >= 0 && d <= 9007199254740992.0 ) || d != std::floor( d ) ) {
      throw JsonError( "JSON: a non-negative whole number is needed" );
    }
    return static_cast<uint64_t>( d );
  }
  bool boolean() const
  {
    want( Kind::Bool, "true or false" );
    return number_ != 0;
  }
  const std::string& string() const
  {
    want( Kind::String, "a string" );
    return text_;
  }
  const std::vector<Json>& array() const
  {
    want( Kind::Array, "an array" );
    return items_;
  }
  const std::map<std::string, Json>& object() const
  {
    want( Kind::Object, "an object" );
    return members_;
  }
  // member of an object; nullptr when absent
  const Json* find( const std::string& key ) const
  {
    const auto& m = object();
    const auto it = m.find( key );
    return it == m.end() ? nullptr : &it->second;
  }
  const Json& operator[]( const std::string& key ) const
  {
    const Json* v = find( key );
    if ( v == nullptr ) {
      throw JsonError( "JSON: member \"" + key + "\" is missing" );
    }
    return *v;
  }

private:
  struct Parser
  {
    std::string_view text;
    size_t at { 0 };

    [[noreturn]] void fail( const char* what ) const { throw JsonError( std::string( "JSON: " ) + what + " at byte " + std::to_string( at ) ); }
    void space()
    {
      while ( at < text.size() && ( text[at] == ' ' || text[at] == '\t' || text[at] == '\n' || text[at] == '\r' ) ) {
        at++;
      }
    }
    bool take( const char c )
    {
      if ( at < text.size() && text[at] == c ) {
        at++;
        return true;
      }
      return false;
    }
    bool word( const std::string_view w )
    {
      if ( text.substr( at, w.size() ) == w ) {
        at += w.size();
        return true;
      }
      return false;
    }

    Json value( const int depth )
    {
      if ( depth > 64 ) {
        fail( "nesting too deep" );
      }
      space();
      if ( at >= text.size() ) {
        fail( "value expected" );
      }
      Json v;
      const char c = text[at];
      if ( c == '{' ) {
        at++;
        v.kind_ = Kind::Object;
        space();
        if ( take( '}' ) ) {
          return v;
        }
        do {
          space();
          std::string key = quoted();
          space();
          if ( !take( ':' ) ) {
            fail( "':' expected" );
          }
          v.members_[std::move( key )] = value( depth + 1 );
          space();
        } while ( take( ',' ) );
        if ( !take( '}' ) ) {
          fail( "'}' expected" );
        }
      } else if ( c == '[' ) {
        at++;
        v.kind_ = Kind::Array;
        space();
        if ( take( ']' ) ) {
          return v;
        }
        do {
          v.items_.push_back( value( depth + 1 ) );
          space();
        } while ( take( ',' ) );
        if ( !take( ']' ) ) {
          fail( "']' expected" );
        }
      } else if ( c == '"' ) {
        v.kind_ = Kind::String;
        v.text_ = quoted();
      } else if ( word( "true" ) ) {
        v.kind_ = Kind::Bool;
        v.number_ = 1;
      } else if ( word( "false" ) ) {
        v.kind_ = Kind::Bool;
      } else if ( !word( "null" ) ) {
        v.kind_ = Kind::Number;
        size_t end = at;
        while ( end < text.size() && ( ( text[end] >= '0' && text[end] <= '9' ) || text[end] == '-' || text[end] == '+' || text[end] == '.' || text[end] == 'e' || text[end] == 'E' ) ) {
          end++;
        }
        const std::string digits( text.substr( at, end - at ) );
        char* stop = nullptr;
        v.number_ = digits.empty() || digits[0] == '+' ? 0.0 : std::strtod( digits.c_str(), &stop );
        if ( stop == nullptr || *stop != '\0' || stop == digits.c_str() ) {
          fail( "value expected" );
        }
        at = end;
      }
      return v;
    }

    unsigned hex4()
    {
      unsigned u = 0;
      for ( int i = 0; i < 4; i++, at++ ) {
        const char c = at < text.size() ? text[at] : '\0';
        u = u * 16;
        if ( c >= '0' && c <= '9' ) {
          u += c - '0';
        } else if ( c >= 'a' && c <= 'f' ) {
          u += c - 'a' + 10;
        } else if ( c >= 'A' && c <= 'F' ) {
          u += c - 'A' + 10;
        } else {
          fail( "four hexadecimal digits expected" );
        }
      }
      return u;
    }

    std::string quoted()
    {
      if ( !take( '"' ) ) {
        fail( "string expected" );
      }
      std::string out;
      while ( true ) {
        if ( at >= text.size() ) {
          fail( "unterminated string" );
        }
        const char c = text[at++];
        if ( c == '"' ) {
          return out;
        }
        if ( c != '\\' ) {
          out += c;
          continue;
        }
        const char e = at < text.size() ? text[at++] : '\0';
        switch ( e ) {
          case '"':
          case '\\':
          case '/': out += e; break;
          case 'b': out += '\b'; break;
          case 'f': out += '\f'; break;
          case 'n': out += '\n'; break;
          case 'r': out += '\r'; break;
          case 't': out += '\t'; break;
          case 'u': {
            unsigned u = hex4();
            if ( u >= 0xd800 && u < 0xdc00 && word( "\\u" ) ) {
              u = 0x10000 + ( ( u - 0xd800 ) << 10 ) + ( hex4() - 0xdc00 );
            }
            if ( u < 0x80 ) {
              out += static_cast<char>( u );
            } else if ( u < 0x800 ) {
              out += static_cast<char>( 0xc0 | ( u >> 6 ) );
              out += static_cast<char>( 0x80 | ( u & 63 ) );
            } else if ( u < 0x10000 ) {
              out += static_cast<char>( 0xe0 | ( u >> 12 ) );
              out += static_cast<char>( 0x80 | ( ( u >> 6 ) & 63 ) );
              out += static_cast<char>( 0x80 | ( u & 63 ) );
            } else {
              out += static_cast<char>( 0xf0 | ( u >> 18 ) );
              out += static_cast<char>( 0x80 | ( ( u >> 12 ) & 63 ) );
              out += static_cast<char>( 0x80 | ( ( u >> 6 ) & 63 ) );
              out += static_cast<char>( 0x80 | ( u & 63 ) );
            }
            break;
          }
          default: fail( "unknown escape" );
        }
      }
    }
  };

  void want( const Kind k, const char* what ) const
  {
    if ( kind_ != k ) {
      throw JsonError( std::string( "JSON: " ) + what + " is needed" );
    }
  }

  Kind kind_ { Kind::Null };
  double number_ { 0 };
  std::string text_ {};
  std::vector<Json> items_ {};
  std::map<std::string, Json> members_ {};
};

} // namespace glint
